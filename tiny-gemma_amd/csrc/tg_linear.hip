// Products with bfloat16 or float32 weights: packing, one-row products (decode) and tiled products (prefill).
// Layout and number formats: tg_linear.h.

#include "tg_linear.h"

namespace {

// ---- packing (load time) -----------------------------------------------------------------------------------------------
__device__ __forceinline__ float pack_read(const TgPack &p, int i, int j) {
	const int gi = i / p.gp, ri = i - gi * p.gp, gj = j / p.kgp, rj = j - gj * p.kgp;
	const int r = gi * p.g + ri, c = gj * p.kg + rj;
	if (ri >= p.g || rj >= p.kg || r >= p.rsrc || c >= p.ksrc) return 0.0f;
	const size_t at = p.transpose ? (size_t)c * p.src_ld + r : (size_t)r * p.src_ld + c;
	return (p.src_f32 ? ((const float *)p.src)[at] : (float)((const __bf16 *)p.src)[at]) + p.add;
}

template <class TR>
__global__ __launch_bounds__(256) void pack_kernel(typename TR::T *dst, int k, TgPack p) {
	const long long total = (long long)p.rows * p.cols;
	for (long long e = (long long)blockIdx.x * 256 + threadIdx.x; e < total; e += (long long)gridDim.x * 256) {
		const int i = (int)(e / p.cols), j = (int)(e - (long long)i * p.cols);
		const int row = (i / 16) * 16 * p.frag_step + p.frag_off * 16 + i % 16;
		const size_t frag = (size_t)(row / 16) * (k / TR::KF) + j / TR::KF;
		const int lane = row % 16 + 16 * ((j % TR::KF) / TR::KV);
		dst[frag * 64 * TR::KV + lane * TR::KV + j % TR::KV] = (typename TR::T)pack_read(p, i, j);
	}
}

__global__ __launch_bounds__(256) void unpack_f32_kernel(float *dst, int ld, TgPack p) {
	const long long total = (long long)p.rows * p.cols;
	for (long long e = (long long)blockIdx.x * 256 + threadIdx.x; e < total; e += (long long)gridDim.x * 256) {
		const int i = (int)(e / p.cols), j = (int)(e - (long long)i * p.cols);
		dst[(size_t)i * ld + j] = pack_read(p, i, j);
	}
}

// ---- one-row products ----------------------------------------------------------------------------------------------------
constexpr int NT = 256;

// Experts by rank: expert e is chosen when fewer than `top` experts have a larger choice score (or the same one and a
// lower index).  s_sel / s_val (LDS, top entries): the chosen experts in rank order and their scores.
__device__ __forceinline__ void choose_experts(const float *logits, const float *correction, int E, int top, float *s_choice, int *s_sel,
                                               float *s_val) {
	const int E4 = (E + 3) & ~3;  // s_choice has room for a multiple of four
	for (int e = threadIdx.x; e < E4; e += NT) s_choice[e] = e < E ? tg_sigmoid(logits[e]) + correction[e] : -INFINITY;
	__syncthreads();
	for (int e = threadIdx.x; e < E; e += NT) {
		const float c = s_choice[e];
		int rank = 0;
		for (int o = 0; o < E4; o += 4) {
			const f32x4_t co = tg_load4(s_choice + o);
#pragma unroll
			for (int i = 0; i < 4; i++) rank += (co[i] > c || (co[i] == c && o + i < e)) ? 1 : 0;
		}
		if (rank < top) {
			s_sel[rank] = e;
			s_val[rank] = tg_sigmoid(logits[e]);
		}
	}
	__syncthreads();
}

// A launch is a chain of dependent memory round trips, so every prologue requests all of its inputs before it uses one
// (clamped indices, no loads under branches), and the first round of the weight stream right behind them: waits are in
// order, the prologue's arithmetic then runs while the weights are on their way.

// NTL: tiles per wave (2: a gate|up pair); KW: waves that share a tile's K (4), or 1: every wave has tiles of its own;
// U: fragments in flight per lane and tile
template <class TR, int PRO, int EPI, int NTL, int KW, int U>
__global__ __launch_bounds__(NT) void vec_kernel(TgVec p) {
	typedef typename TR::T T;
	typedef typename TR::Frag Frag;
	extern __shared__ __align__(16) unsigned char smem[];
	T *xs = reinterpret_cast<T *>(smem);
	__shared__ float s_red[4][NTL * 16];
	__shared__ float s_misc[64];
	const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
	const int part = blockIdx.y, z = blockIdx.z;
	const int per = (p.kfrags + p.ksplit - 1) / p.ksplit;
	const int kb = part * per, ke = min(p.kfrags, kb + per), nk = max(ke - kb, 0);
	const int k0 = kb * TR::KF, kn = nk * TR::KF;

	int zw = z;
	if constexpr (PRO == TG_VP_EXPERT) {
		// LDS: choice scores [experts, padded] | selected [top] | their scores [top] behind the vector
		float *s_choice = reinterpret_cast<float *>(smem + sizeof(T) * (size_t)(per + KW * U) * TR::KF);
		int *s_sel = reinterpret_cast<int *>(s_choice + ((p.experts + 3) & ~3));
		float *s_val = reinterpret_cast<float *>(s_sel + p.top);
		choose_experts(p.logits, p.correction, p.experts, p.top, s_choice, s_sel, s_val);
		zw = s_sel[z];
		if (blockIdx.x == 0 && part == 0 && z == 0) {
			for (int k = tid; k < p.top; k += NT) {
				float sum = 0.0f;
				for (int o = 0; o < p.top; o++) sum += s_val[o];
				p.sel[k] = s_sel[k];
				p.wgt[k] = s_val[k] / (sum + 1e-20f) * p.rscale;
			}
		}
	}
	if constexpr (EPI == TG_VE_WEIGHTED) zw = p.sel[z];

	const int group = KW == 4 ? (int)blockIdx.x : (int)blockIdx.x * 4 + w;  // tile group of this wave
	const bool live = group * NTL < p.ntiles;
	const int tile0 = live ? group * NTL : 0, tiles_here = min(NTL, p.ntiles - tile0);
	const Frag *W = reinterpret_cast<const Frag *>(p.W) + ((size_t)zw * p.zfrags + (size_t)tile0 * p.kfrags) * 64 + lane;
	const int step = KW, kf0 = kb + (KW == 4 ? w : 0);
	Frag wr[NTL][U];
	auto load = [&](int kf) {
#pragma unroll
		for (int u = 0; u < U; u++) {
			const int kk = kf + u * step, kc = min(kk, p.kfrags - 1);
#pragma unroll
			for (int t = 0; t < NTL; t++) {
				const Frag *at = W + ((size_t)(t < tiles_here ? t : 0) * p.kfrags + kc) * 64;
				// a head is read once per token: past the caches, which keep the layers' matrices
				wr[t][u] = KW == 1 ? __builtin_nontemporal_load(at) : *at;
			}
		}
	};

	// the vector's prologue: elements [k0, k0 + kn), then zeros that the surplus steps of the last round multiply
	if constexpr (PRO == TG_VP_PLAIN || PRO == TG_VP_EXPERT) {
		const float *x = p.x + (PRO == TG_VP_PLAIN ? (size_t)z * p.x_zstride : 0) + k0;
		for (int b = 0; b == 0 || b < kn; b += 8 * NT) {
			f32x4_t v[2];
#pragma unroll
			for (int i = 0; i < 2; i++) v[i] = tg_load4(x + min(b + 4 * (tid + i * NT), max(kn - 4, 0)));
			if (b == 0) load(kf0);
#pragma unroll
			for (int i = 0; i < 2; i++)
				if (b + 4 * (tid + i * NT) < kn) tg_store4(xs + b + 4 * (tid + i * NT), v[i]);
		}
	} else if constexpr (PRO == TG_VP_DYT) {
		int row = 0;
		if (p.embed) {
			row = p.ctr[4];
			row = row < 0 ? 0 : (row >= p.vocab ? p.vocab - 1 : row);
		}
		// two elements per lane and pass; the padding behind the vector is zero in x, the parts, the norm and the table
		constexpr int PER = 4, PQ = 8;
		for (int b = 0; b == 0 || b < kn; b += 2 * PER * NT) {
			float2 x[PER], nw[PER], nb[PER], pq[PER][PQ];
			int c[PER];
#pragma unroll
			for (int i = 0; i < PER; i++) {
				const int j = b + 2 * (tid + i * NT);
				c[i] = k0 + min(j, max(kn - 2, 0));
				if (p.embed) {
					const unsigned u = *reinterpret_cast<const unsigned *>((const __bf16 *)p.embed + (size_t)row * p.embed_ld + c[i]);
					x[i] = float2{__uint_as_float(u << 16), __uint_as_float(u & 0xffff0000u)};
				} else {
					x[i] = *reinterpret_cast<const float2 *>(p.x + c[i]);
				}
				nw[i] = *reinterpret_cast<const float2 *>(p.nw + c[i]);
				nb[i] = *reinterpret_cast<const float2 *>(p.nb + c[i]);
			}
			float2 add[PER];
#pragma unroll
			for (int i = 0; i < PER; i++) add[i] = float2{0.0f, 0.0f};
			for (int q0 = 0; q0 < p.nparts; q0 += PQ) {
#pragma unroll
				for (int q = 0; q < PQ; q++)
#pragma unroll
					for (int i = 0; i < PER; i++)
						pq[i][q] = *reinterpret_cast<const float2 *>(p.pend + (size_t)min(q0 + q, p.nparts - 1) * p.pend_stride + c[i]);
				if (b == 0 && q0 == 0) load(kf0);
#pragma unroll
				for (int q = 0; q < PQ; q++)
					if (q0 + q < p.nparts)
#pragma unroll
						for (int i = 0; i < PER; i++) {
							add[i].x += pq[i][q].x;
							add[i].y += pq[i][q].y;
						}
			}
			if (b == 0 && p.nparts == 0) load(kf0);
#pragma unroll
			for (int i = 0; i < PER; i++) {
				const int j = b + 2 * (tid + i * NT);
				if (p.nparts) {
					x[i].x = x[i].x + p.mult * add[i].x;
					x[i].y = x[i].y + p.mult * add[i].y;
				}
				const float2 h = {tanhf(p.alpha * x[i].x) * nw[i].x + nb[i].x, tanhf(p.alpha * x[i].y) * nw[i].y + nb[i].y};
				if (j < kn) {
					xs[j] = (T)h.x;
					xs[j + 1] = (T)h.y;
					if (blockIdx.x == 0 && z == 0) {
						if (p.x_out) *reinterpret_cast<float2 *>(p.x_out + c[i]) = x[i];
						if (p.h_out) *reinterpret_cast<float2 *>(p.h_out + c[i]) = h;
					}
				}
			}
		}
	} else if constexpr (PRO == TG_VP_RMS) {
		// The whole vector in every workgroup (ksplit is 1): four elements per lane and pass; the first RP passes stay in
		// registers, the rest goes through LDS.  The padding is zero in x, the parts, the weights and the table.
		constexpr int RP = 2, PQ = 8;
		int row = 0;
		if (p.embed) {
			row = p.ctr[4];
			row = row < 0 ? 0 : (row >= p.vocab ? p.vocab - 1 : row);
		}
		float *sv = reinterpret_cast<float *>(smem + sizeof(T) * (size_t)(per + KW * U) * TR::KF);  // [kn], wider vectors only
		const int npass = (kn + 4 * NT - 1) / (4 * NT);
		f32x4_t x[RP], add[RP], nw[RP], pw[RP];
		auto at = [&](int i) { return min(4 * (tid + i * NT), kn - 4); };
		auto source = [&](int c) {
			f32x4_t v;
			if (p.embed) {
				v = tg_load4((const __bf16 *)p.embed + (size_t)row * p.embed_ld + c);
#pragma unroll
				for (int e = 0; e < 4; e++) v[e] *= p.embed_scale;
			} else {
				v = tg_load4(p.x + c);
			}
			return v;
		};
		auto parts = [&](int c) {
			f32x4_t r = {0, 0, 0, 0};
			for (int q0 = 0; q0 < p.nparts; q0 += PQ) {
				f32x4_t v[PQ];
#pragma unroll
				for (int q = 0; q < PQ; q++) v[q] = tg_load4(p.pend + (size_t)min(q0 + q, p.nparts - 1) * p.pend_stride + c);
#pragma unroll
				for (int q = 0; q < PQ; q++)
					if (q0 + q < p.nparts)
#pragma unroll
						for (int e = 0; e < 4; e++) r[e] += v[q][e];
			}
			return r;
		};
		auto total = [&](float v, int slot) {
			v = tg_wave_sum(v);
			if (lane == 0) s_misc[slot + w] = v;
			__syncthreads();
			return (s_misc[slot] + s_misc[slot + 1]) + (s_misc[slot + 2] + s_misc[slot + 3]);
		};
#pragma unroll
		for (int i = 0; i < RP; i++) {
			const int c = at(i);
			x[i] = source(c);
			nw[i] = tg_load4(p.nw + c);
			if (p.nparts) pw[i] = p.post ? tg_load4(p.post + c) : f32x4_t{p.mult, p.mult, p.mult, p.mult};
		}
		if (p.nparts) {
#pragma unroll
			for (int i = 0; i < RP; i++) add[i] = parts(at(i));
		}
		load(kf0);
		auto wide = [&](int i, auto &&f) {  // f(column, its four values in LDS)
			for (; i < npass; i++) {
				const int j = 4 * (tid + i * NT);
				if (j < kn) f(j);
			}
		};
		if (p.nparts) {
			float inv = 1.0f;
			if (p.post) {
				float ss = 0.0f;
#pragma unroll
				for (int i = 0; i < RP; i++)
					if (4 * (tid + i * NT) < kn)
#pragma unroll
						for (int e = 0; e < 4; e++) ss = fmaf(add[i][e], add[i][e], ss);
				wide(RP, [&](int j) {
					const f32x4_t v = parts(j);
#pragma unroll
					for (int e = 0; e < 4; e++) ss = fmaf(v[e], v[e], ss);
					tg_store4(sv + j, v);
				});
				inv = 1.0f / sqrtf(total(ss, 0) / (float)p.width + p.eps);
			} else {
				wide(RP, [&](int j) { tg_store4(sv + j, parts(j)); });
			}
#pragma unroll
			for (int i = 0; i < RP; i++)
#pragma unroll
				for (int e = 0; e < 4; e++) x[i][e] += add[i][e] * inv * pw[i][e];
			wide(RP, [&](int j) {
				f32x4_t v = source(j);
				const f32x4_t a = tg_load4(sv + j), b = p.post ? tg_load4(p.post + j) : f32x4_t{p.mult, p.mult, p.mult, p.mult};
#pragma unroll
				for (int e = 0; e < 4; e++) v[e] += a[e] * inv * b[e];
				tg_store4(sv + j, v);
			});
		} else {
			wide(RP, [&](int j) { tg_store4(sv + j, source(j)); });
		}
		float ss = 0.0f;
#pragma unroll
		for (int i = 0; i < RP; i++)
			if (4 * (tid + i * NT) < kn)
#pragma unroll
				for (int e = 0; e < 4; e++) ss = fmaf(x[i][e], x[i][e], ss);
		wide(RP, [&](int j) {
			const f32x4_t v = tg_load4(sv + j);
#pragma unroll
			for (int e = 0; e < 4; e++) ss = fmaf(v[e], v[e], ss);
		});
		const float inv = 1.0f / sqrtf(total(ss, 4) / (float)p.width + p.eps);
		const bool first = blockIdx.x == 0 && z == 0;
		auto finish = [&](int j, f32x4_t v, f32x4_t n) {
			f32x4_t h;
#pragma unroll
			for (int e = 0; e < 4; e++) h[e] = v[e] * inv * n[e];
			tg_store4(xs + j, h);
			if (first && p.x_out) tg_store4(p.x_out + j, v);
			if (first && p.h_out) tg_store4(p.h_out + j, h);
		};
#pragma unroll
		for (int i = 0; i < RP; i++)
			if (4 * (tid + i * NT) < kn) finish(4 * (tid + i * NT), x[i], nw[i]);
		wide(RP, [&](int j) { finish(j, tg_load4(sv + j), tg_load4(p.nw + j)); });
	} else if constexpr (PRO == TG_VP_HEADNORM) {
		// head by head, a wave each, four elements per lane and pass: sum of squares, then the head's elements that lie in
		// this part of K
		const int h_lo = k0 / p.vdimp, h_hi = min((k0 + kn - 1) / p.vdimp, p.heads16 - 1), vl = p.vdimp - 4;
		bool first = true;
		for (int a = h_lo + w; a <= h_hi; a += 4) {
			const float *o = p.x + (size_t)a * p.vdimp, *g = p.gate + (size_t)a * p.vdimp;
			const f32x4_t o0 = tg_load4(o + min(4 * lane, vl)), g0 = tg_load4(g + min(4 * lane, vl)), w0 = tg_load4(p.nw + min(4 * lane, vl));
			if (first) load(kf0);
			first = false;
			float ss = 0.0f;
			for (int v = 4 * lane; v < p.vdimp; v += 256) {  // the padding is zero
				const f32x4_t ov = v < 256 ? o0 : tg_load4(o + v);
#pragma unroll
				for (int e = 0; e < 4; e++) ss = fmaf(ov[e], ov[e], ss);
			}
			ss = tg_wave_sum(ss);
			const float inv = 1.0f / sqrtf(ss / (float)p.vdim + p.eps);
			for (int v = 4 * lane; v < p.vdimp; v += 256) {
				const f32x4_t ov = v < 256 ? o0 : tg_load4(o + v), gv = v < 256 ? g0 : tg_load4(g + v), wv = v < 256 ? w0 : tg_load4(p.nw + v);
				const int j = a * p.vdimp + v - k0;
				f32x4_t r;
#pragma unroll
				for (int e = 0; e < 4; e++) r[e] = ov[e] * inv * wv[e] * (p.gate_sigmoid ? tg_sigmoid(gv[e]) : tg_silu(gv[e]));
				if (j >= 0 && j < kn) tg_store4(xs + j, r);
			}
		}
		if (first) load(kf0);
		for (int j = tid; j < kn; j += NT)
			if ((k0 + j) / p.vdimp >= p.heads16) xs[j] = (T)0.0f;
	} else if constexpr (PRO == TG_VP_MERGE_HEADS) {
		// a row of 16 lanes per head: the factors of its partials; then element by element
		__shared__ float s_f[TG_VEC_MERGE_HEADS_MAX][TG_VEC_MERGE_MAX];
		const int g16 = (p.group + 15) / 16 * 16, bl = min(lane & 15, p.nmerge - 1);
		auto padded = [&](int h) { const int g = h / p.group; return g * g16 + h - g * p.group; };
		const int h_lo = min(k0 / p.vdimp, p.heads - 1), h_hi = min((k0 + max(kn, 1) - 1) / p.vdimp, p.heads - 1);
		auto column = [&](int j) {
			const int k = k0 + j, h = min(k / p.vdimp, p.heads - 1);
			return p.part_acc + (size_t)padded(h) * p.x_zstride + min(k - h * p.vdimp, p.vdimp - 1);
		};
		const size_t step_b = (size_t)p.heads16 * p.x_zstride;
		const int ha = min(h_lo + 4 * w + (lane >> 4), h_hi);
		float2 ml = *reinterpret_cast<const float2 *>(p.part_ml + ((size_t)bl * p.heads16 + padded(ha)) * 2);
		float a[TG_VEC_MERGE_MAX];
		const float *pa = column(min(tid, max(kn - 1, 0)));
#pragma unroll
		for (int b = 0; b < TG_VEC_MERGE_MAX; b++) a[b] = pa[(size_t)min(b, p.nmerge - 1) * step_b];
		load(kf0);
		const bool in = (lane & 15) < p.nmerge;
		for (int hb = h_lo; hb <= h_hi; hb += 16) {
			const int h = min(hb + 4 * w + (lane >> 4), h_hi);
			if (hb != h_lo) ml = *reinterpret_cast<const float2 *>(p.part_ml + ((size_t)bl * p.heads16 + padded(h)) * 2);
			const float m = tg_row16_max(in ? ml.x : -INFINITY);
			const float f = in ? expf(ml.x - m) : 0.0f;
			const float inv = 1.0f / tg_row16_sum(f * ml.y);
			s_f[h - h_lo][lane & 15] = f * inv;
		}
		__syncthreads();
		for (int j = tid; j < kn; j += NT) {
			const int h = (k0 + j) / p.vdimp;
			if (j != tid) {
				pa = column(j);
#pragma unroll
				for (int b = 0; b < TG_VEC_MERGE_MAX; b++) a[b] = pa[(size_t)min(b, p.nmerge - 1) * step_b];
			}
			float r = 0.0f;
			if (h < p.heads)
#pragma unroll
				for (int b = 0; b < TG_VEC_MERGE_MAX; b++) r = fmaf(s_f[h - h_lo][b], a[b], r);
			xs[j] = (T)r;
		}
	} else {  // MERGE: at most 16 partials
		const int bl = min(lane & 15, p.nmerge - 1);
		const float2 ml = *reinterpret_cast<const float2 *>(p.part_ml + ((size_t)bl * p.heads16 + z) * 2);
		float a[TG_VEC_MERGE_MAX];
		const float *pa = p.part_acc + (size_t)z * p.x_zstride + k0;
#pragma unroll
		for (int b = 0; b < TG_VEC_MERGE_MAX; b++)
			a[b] = pa[(size_t)min(b, p.nmerge - 1) * p.heads16 * p.x_zstride + min(tid, max(kn - 1, 0))];
		load(kf0);
		const bool in = (lane & 15) < p.nmerge;
		const float m = tg_row16_max(in ? ml.x : -INFINITY);
		const float f = in ? expf(ml.x - m) : 0.0f;
		const float inv = 1.0f / tg_row16_sum(f * ml.y);
		if (tid < 16) s_misc[tid] = f * inv;
		__syncthreads();
		for (int j = tid; j < kn; j += NT) {
			float r = 0.0f;
#pragma unroll
			for (int b = 0; b < TG_VEC_MERGE_MAX; b++) {
				if (j != tid) a[b] = pa[(size_t)min(b, p.nmerge - 1) * p.heads16 * p.x_zstride + j];
				r = fmaf(s_misc[b], a[b], r);
			}
			xs[j] = (T)r;
		}
	}
	for (int j = kn + tid; j < kn + KW * U * TR::KF; j += NT) xs[j] = (T)0.0f;
	__syncthreads();

	f32x4_t acc[NTL];
#pragma unroll
	for (int t = 0; t < NTL; t++) acc[t] = f32x4_t{0, 0, 0, 0};
	const T *xl = xs + (lane >> 4) * TR::KV;
	for (int kf = kf0; kf < ke; kf += step * U) {
		Frag cur[NTL][U];
#pragma unroll
		for (int t = 0; t < NTL; t++)
#pragma unroll
			for (int u = 0; u < U; u++) cur[t][u] = wr[t][u];
		if (kf + step * U < ke) load(kf + step * U);
#pragma unroll
		for (int u = 0; u < U; u++) {
			const Frag xf = *reinterpret_cast<const Frag *>(xl + (size_t)(kf + u * step - kb) * TR::KF);
#pragma unroll
			for (int t = 0; t < NTL; t++) acc[t] = TR::mma(xf, cur[t][u], acc[t]);
		}
	}
	// all 16 rows of the first operand are the vector: element 0 of lane l is output l % 16 of the tile
	if constexpr (KW == 4) {
		if (lane < 16) {
#pragma unroll
			for (int t = 0; t < NTL; t++) s_red[w][t * 16 + lane] = acc[t][0];
		}
		__syncthreads();
		if (tid < 16) {
			float v[NTL];
#pragma unroll
			for (int t = 0; t < NTL; t++) v[t] = (s_red[0][t * 16 + tid] + s_red[1][t * 16 + tid]) + (s_red[2][t * 16 + tid] + s_red[3][t * 16 + tid]);
			float *y = p.y + (size_t)part * p.part_stride + (size_t)z * p.y_zstride;
			if constexpr (EPI == TG_VE_SWIGLU) {
				y[group * 16 + tid] = tg_silu(v[0]) * v[NTL - 1];
			} else {
				float r = v[0];
				if constexpr (EPI == TG_VE_STORE) {
					if (p.bias) {
						r += p.bias[group * NTL * 16 + tid];
						if constexpr (NTL == 2) {
							if (group * 2 + 1 < p.ntiles) v[1] += p.bias[group * 32 + 16 + tid];
						}
					}
				}
				if constexpr (EPI == TG_VE_GELU) r = tg_gelu(r);
				if constexpr (EPI == TG_VE_GATE) r *= tg_sigmoid(p.gate[z]);
				if constexpr (EPI == TG_VE_WEIGHTED) r *= p.wgt[z];
				y[group * NTL * 16 + tid] = r;
				if constexpr (NTL == 2) {
					if (group * 2 + 1 < p.ntiles) y[group * 32 + 16 + tid] = v[1];
				}
				if constexpr (EPI == TG_VE_LOGITS) {
					float bv = group * 16 + tid < p.nout ? r : -INFINITY;
					int bi = group * 16 + tid;
#pragma unroll
					for (int o = 8; o > 0; o >>= 1) {
						const float ov = __shfl_xor(bv, o, 16);
						const int oi = __shfl_xor(bi, o, 16);
						if (ov > bv || (ov == bv && oi < bi)) { bv = ov; bi = oi; }
					}
					if (tid == 0) { p.blk_val[blockIdx.x] = bv; p.blk_idx[blockIdx.x] = bi; }
				}
			}
		}
	} else {
		if (lane < 16) {
			const int o = group * 16 + lane;
			float r = acc[0][0];
			if constexpr (EPI == TG_VE_STORE) {
				if (p.bias && live) r += p.bias[o];
			}
			if (live) p.y[(size_t)z * p.y_zstride + o] = r;
			if constexpr (EPI == TG_VE_LOGITS) s_red[w][lane] = live && o < p.nout ? r : -INFINITY;
		}
		if constexpr (EPI == TG_VE_LOGITS) {
			__syncthreads();
			if (tid < 64) {
				float bv = s_red[tid >> 4][tid & 15];
				int bi = (int)blockIdx.x * 64 + tid;
#pragma unroll
				for (int o = 32; o > 0; o >>= 1) {
					const float ov = __shfl_xor(bv, o, 64);
					const int oi = __shfl_xor(bi, o, 64);
					if (ov > bv || (ov == bv && oi < bi)) { bv = ov; bi = oi; }
				}
				if (tid == 0) { p.blk_val[blockIdx.x] = bv; p.blk_idx[blockIdx.x] = bi; }
			}
		}
	}
}

bool vec_wide(const TgVec &v, int epi) { return (epi == TG_VE_STORE || epi == TG_VE_LOGITS) && v.ksplit == 1 && v.nz == 1 && v.ntiles >= 2048; }

// Two tiles per workgroup where one each would be two workgroups per compute unit and more: the prologue (with its reads of
// the parts of the residual) is done half as often.
bool vec_pairs(const TgVec &v, int epi) { return epi == TG_VE_STORE && v.nparts > 0 && v.nz == 1 && v.ksplit == 1 && v.ntiles >= 448; }

// the norm's vector beyond what the registers of a workgroup hold
size_t rms_lds(int pro, int k) { return pro == TG_VP_RMS && k > 8 * NT ? sizeof(float) * (size_t)k : 0; }

template <class TR, int PRO, int EPI>
void launch_vec_t(const TgVec &v, hipStream_t s) {
	constexpr int NTL = EPI == TG_VE_SWIGLU ? 2 : 1;
	const int per = (v.kfrags + v.ksplit - 1) / v.ksplit;
	if constexpr ((PRO == TG_VP_DYT || PRO == TG_VP_RMS) && EPI == TG_VE_STORE) {
		if (!vec_wide(v, EPI) && vec_pairs(v, EPI)) {
			const int n = (per + 3) / 4;
			auto lds = [&](int pad) { return sizeof(typename TR::T) * (size_t)(per + pad) * TR::KF + rms_lds(PRO, per * TR::KF); };
			const dim3 grid((unsigned)tg_vec_blocks(v, EPI), (unsigned)v.ksplit, (unsigned)v.nz);
			if (n <= 6) hipLaunchKernelGGL((vec_kernel<TR, PRO, EPI, 2, 4, 6>), grid, dim3(NT), lds(24), s, v);
			else hipLaunchKernelGGL((vec_kernel<TR, PRO, EPI, 2, 4, 8>), grid, dim3(NT), lds(32), s, v);
			return;
		}
	}
	const unsigned bx = (unsigned)tg_vec_blocks(v, EPI);
	auto lds = [&](int pad) {
		size_t b = sizeof(typename TR::T) * (size_t)(per + pad) * TR::KF;
		b += rms_lds(PRO, per * TR::KF);
		if (PRO == TG_VP_EXPERT) b += sizeof(float) * (size_t)(((v.experts + 3) & ~3) + 2 * v.top);
		return b;
	};
	if constexpr (EPI == TG_VE_STORE || EPI == TG_VE_LOGITS) {
		if (vec_wide(v, EPI)) {
			hipLaunchKernelGGL((vec_kernel<TR, PRO, EPI, 1, 1, 8>), dim3(bx, 1, 1), dim3(NT), lds(8), s, v);
			return;
		}
	}
	// fragments in flight: all of a wave's where they fit, else in as few equal rounds as possible
	const dim3 grid(bx, (unsigned)v.ksplit, (unsigned)v.nz);
	const int n = (per + 3) / 4;
	if (n <= 2) hipLaunchKernelGGL((vec_kernel<TR, PRO, EPI, NTL, 4, 2>), grid, dim3(NT), lds(8), s, v);
	else if (n <= 4) hipLaunchKernelGGL((vec_kernel<TR, PRO, EPI, NTL, 4, 4>), grid, dim3(NT), lds(16), s, v);
	else if (n <= 6 || (n > 9 && n <= 12)) hipLaunchKernelGGL((vec_kernel<TR, PRO, EPI, NTL, 4, 6>), grid, dim3(NT), lds(24), s, v);
	else if (n <= 8 || (n > 12 && n <= 16) || (n > 18 && n <= 24)) hipLaunchKernelGGL((vec_kernel<TR, PRO, EPI, NTL, 4, 8>), grid, dim3(NT), lds(32), s, v);
	else hipLaunchKernelGGL((vec_kernel<TR, PRO, EPI, NTL, 4, 9>), grid, dim3(NT), lds(36), s, v);
}

template <class TR>
void launch_vec_dt(const TgVec &v, int pro, int epi, hipStream_t s) {
	if (pro == TG_VP_PLAIN && epi == TG_VE_STORE) launch_vec_t<TR, TG_VP_PLAIN, TG_VE_STORE>(v, s);
	else if (pro == TG_VP_DYT && epi == TG_VE_STORE) launch_vec_t<TR, TG_VP_DYT, TG_VE_STORE>(v, s);
	else if (pro == TG_VP_DYT && epi == TG_VE_LOGITS) launch_vec_t<TR, TG_VP_DYT, TG_VE_LOGITS>(v, s);
	else if (pro == TG_VP_RMS && epi == TG_VE_STORE) launch_vec_t<TR, TG_VP_RMS, TG_VE_STORE>(v, s);
	else if (pro == TG_VP_RMS && epi == TG_VE_GELU) launch_vec_t<TR, TG_VP_RMS, TG_VE_GELU>(v, s);
	else if (pro == TG_VP_RMS && epi == TG_VE_LOGITS) launch_vec_t<TR, TG_VP_RMS, TG_VE_LOGITS>(v, s);
	else if (pro == TG_VP_MERGE && epi == TG_VE_STORE) launch_vec_t<TR, TG_VP_MERGE, TG_VE_STORE>(v, s);
	else if (pro == TG_VP_MERGE_HEADS) launch_vec_t<TR, TG_VP_MERGE_HEADS, TG_VE_STORE>(v, s);
	else if (pro == TG_VP_HEADNORM) launch_vec_t<TR, TG_VP_HEADNORM, TG_VE_STORE>(v, s);
	else if (pro == TG_VP_MERGE) launch_vec_t<TR, TG_VP_MERGE, TG_VE_GATE>(v, s);
	else if (pro == TG_VP_EXPERT) launch_vec_t<TR, TG_VP_EXPERT, TG_VE_SWIGLU>(v, s);
	else if (pro == TG_VP_PLAIN && epi == TG_VE_GATE) launch_vec_t<TR, TG_VP_PLAIN, TG_VE_GATE>(v, s);
	else launch_vec_t<TR, TG_VP_PLAIN, TG_VE_WEIGHTED>(v, s);
}

// ---- tiled products --------------------------------------------------------------------------------------------------------
// A workgroup computes BM x BN with WM x WN waves of (16 MI) x (16 NI) each.  K advances by two fragments (128 bytes of a
// row) per stage: both operands go global -> registers -> LDS in fragment order (two LDS buffers, two sets of registers: the
// loads of the next two stages are in flight during the matrix instructions of this one), one LDS-only barrier per stage.
template <class TR, int EPI, int WM, int WN, int MI, int NI, bool GROUPED>
__global__ __launch_bounds__(256, 2) void linear_kernel(TgGemm g) {
	typedef typename TR::T T;
	typedef typename TR::Frag Frag;
	constexpr int BM = WM * MI * 16, BN = WN * NI * 16;
	constexpr int AF = BM / 16, BF = BN / 16, NF = 2 * (AF + BF), PW = NF / 4;  // fragments per stage, per wave
	static_assert(NF % 4 == 0 && WM * WN == 4, "four waves share a stage's fragments");
	__shared__ __align__(16) Frag lds[2][NF * 64];
	const int lane = threadIdx.x & 63, w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
	const int ntn = (g.N + BN - 1) / BN;

	// Workgroups go to the 8 XCDs in turn: give each XCD a contiguous run of the tile order, so that the workgroups it
	// runs side by side share weight tiles and activation rows in its L2.  (A list of groups launches as many workgroups
	// as it could have tiles: the run lengths come from the tiles it has.)
	const int mrows = EPI == TG_GE_TRANS ? g.rows_out : g.M;
	const int ntm = GROUPED ? *g.ntiles : (mrows + BM - 1) / BM;
	int b;
	{
		const int total = ntm * ntn, q = total >> 3, r = total & 7, x = (int)blockIdx.x & 7, i = (int)blockIdx.x >> 3;
		if (i >= q + (x < r ? 1 : 0)) return;
		b = x * q + min(x, r) + i;
	}
	int m0, m1, tn;
	const Frag *W = reinterpret_cast<const Frag *>(g.W);
	if constexpr (GROUPED) {
		const int t = b / ntn;
		tn = b - t * ntn;
		const int4 tile = g.tiles[t];
		m0 = tile.y;
		m1 = tile.z;
		W += (size_t)tile.x * g.group_frags * 64;
	} else {
		tn = b / ntm;
		m0 = (b - tn * ntm) * BM;
		m1 = g.M;
	}
	const int kfr = g.K / TR::KF, nst = kfr / 2, nfr = g.N / 16;

	// this wave's fragments of a stage: f = w * PW + i; the first 2 AF are A (row tile f / 2, k half f % 2), then B
	// (addresses: a base that the wave shares, 32-bit offsets per lane; operands are below 4 GiB)
	const unsigned char *base[PW];
	unsigned off[PW];
	int adv[PW];
#pragma unroll
	for (int i = 0; i < PW; i++) {
		const int f = w * PW + i;
		if (f < 2 * AF) {
			int r = min(m0 + (f >> 1) * 16 + (lane & 15), m1 - 1);
			if (g.row_src) r = g.row_src[r];
			base[i] = reinterpret_cast<const unsigned char *>(g.A) + (f & 1) * 64;
			off[i] = (unsigned)r * (unsigned)(g.lda * (int)sizeof(T)) + (unsigned)(lane >> 4) * 16u;
			adv[i] = 128;
		} else {
			const int fb = f - 2 * AF, nf = min(tn * BF + (fb >> 1), nfr - 1);
			base[i] = reinterpret_cast<const unsigned char *>(W + ((size_t)nf * kfr + (fb & 1)) * 64);
			off[i] = (unsigned)lane * 16u;
			adv[i] = 2048;
		}
	}
	Frag st[2][PW];
	auto fetch = [&](int set, int s) {
		s = min(s, nst - 1);
#pragma unroll
		for (int i = 0; i < PW; i++) st[set][i] = *reinterpret_cast<const Frag *>(base[i] + (size_t)s * adv[i] + off[i]);
	};
	auto put = [&](int set) {
#pragma unroll
		for (int i = 0; i < PW; i++) lds[set][(w * PW + i) * 64 + lane] = st[set][i];
	};
	const int wm = w / WN, wn = w - wm * WN;
	f32x4_t acc[MI][NI];
#pragma unroll
	for (int i = 0; i < MI; i++)
#pragma unroll
		for (int j = 0; j < NI; j++) acc[i][j] = f32x4_t{0, 0, 0, 0};

	// Two sets of operand registers as well: the LDS reads of one half of a stage are in flight during the matrix
	// instructions of the half before it.
	Frag fa[2][MI], fb[2][NI];
	auto read = [&](int kh, int par) {
#pragma unroll
		for (int i = 0; i < MI; i++) fa[kh][i] = lds[par][((wm * MI + i) * 2 + kh) * 64 + lane];
#pragma unroll
		for (int j = 0; j < NI; j++) fb[kh][j] = lds[par][(2 * AF + (wn * NI + j) * 2 + kh) * 64 + lane];
	};
	auto multiply = [&](int kh) {
#pragma unroll
		for (int i = 0; i < MI; i++)
#pragma unroll
			for (int j = 0; j < NI; j++)
				acc[i][j] = EPI == TG_GE_TRANS ? TR::mma(fa[kh][i], fb[kh][j], acc[i][j]) : TR::mma(fb[kh][j], fa[kh][i], acc[i][j]);
	};
	fetch(0, 0);
	fetch(1, 1);
	put(0);
	fetch(0, 2);
	tg_lds_barrier();
	read(0, 0);
	// LDS buffer and register set of a stage: its parity
	// (the order is pinned: left to itself the scheduler moves every LDS read down to its use)
	constexpr int MM = MI * NI * (TR::DT == TG_DT_BF16 ? 1 : 4), RD = MI + NI;
	constexpr int MR = MM / 2 / RD > 0 ? MM / 2 / RD : 1, MP = MM / 2 / PW > 0 ? MM / 2 / PW : 1;
	auto stage = [&](int s, int par) {
		read(1, par);
		multiply(0);
		put(par ^ 1);
		fetch(par ^ 1, s + 3);
#pragma unroll
		for (int i = 0; i < RD; i++) {
			__builtin_amdgcn_sched_group_barrier(0x100, 1, 0);        // LDS read
			__builtin_amdgcn_sched_group_barrier(0x008, MR, 0);  // matrix instructions
		}
#pragma unroll
		for (int i = 0; i < PW; i++) {
			__builtin_amdgcn_sched_group_barrier(0x008, MP, 0);
			__builtin_amdgcn_sched_group_barrier(0x200, 1, 0);        // LDS write
			__builtin_amdgcn_sched_group_barrier(0x020, 1, 0);        // global load
		}
		__builtin_amdgcn_sched_barrier(0);
		tg_lds_barrier();
		__builtin_amdgcn_sched_barrier(0);
		read(0, par ^ 1);
		multiply(1);
#pragma unroll
		for (int i = 0; i < RD; i++) {
			__builtin_amdgcn_sched_group_barrier(0x100, 1, 1);
			__builtin_amdgcn_sched_group_barrier(0x008, MM / RD > 0 ? MM / RD : 1, 1);
		}
		__builtin_amdgcn_sched_barrier(0);
	};
	// (pairs without a branch between them: across one, the waits for the older register set would cover the newer one too)
	int s = 0;
	for (; s + 1 < nst; s += 2) {
		stage(s, 0);
		stage(s + 1, 1);
	}
	if (s < nst) stage(s, 0);

	const int lr = lane & 15, lg = lane >> 4;
	if constexpr (EPI == TG_GE_TRANS) {
		// lane: column n = lr, rows m = 4 lg + i, four consecutive keys of a 32-key (bf16) or 16-key (fp32) operand block
#pragma unroll
		for (int i = 0; i < MI; i++)
#pragma unroll
			for (int j = 0; j < NI; j++) {
				const int n = tn * BN + (wn * NI + j) * 16 + lr, m = m0 + (wm * MI + i) * 16 + 4 * lg;
				if (n >= g.N || m >= g.rows_out) continue;
				int at = m;
				if constexpr (TR::DT == TG_DT_BF16) at = (m & ~31) + lg * 8 + ((m >> 4) & 1) * 4;
				tg_store4((T *)g.C + (size_t)n * g.ldc + at, acc[i][j]);
			}
	} else {
		// lane: row m = lr, columns n = 4 lg + i
#pragma unroll
		for (int i = 0; i < MI; i++) {
			const int m = m0 + (wm * MI + i) * 16 + lr;
			if (m >= m1) continue;
			if constexpr (EPI == TG_GE_SWIGLU) {
#pragma unroll
				for (int j = 0; j < NI; j += 2) {
					const int n = tn * BN + (wn * NI + j) * 16;  // of the interleaved rows
					if (n >= g.N) continue;
					f32x4_t r;
#pragma unroll
					for (int e = 0; e < 4; e++) r[e] = tg_silu(acc[i][j][e]) * acc[i][j + 1][e];
					tg_store4((T *)g.C + (size_t)m * g.ldc + n / 2 + 4 * lg, r);
				}
			} else {
#pragma unroll
				for (int j = 0; j < NI; j++) {
					const int n = tn * BN + (wn * NI + j) * 16 + 4 * lg;
					if (n >= g.N) continue;
					if constexpr (EPI == TG_GE_STORE) {
						if (g.bias && n < g.n_split) {
							const f32x4_t b = tg_load4(g.bias + n);
#pragma unroll
							for (int e = 0; e < 4; e++) acc[i][j][e] += b[e];
						}
						if (n < g.n_split) tg_store4((T *)g.C + (size_t)m * g.ldc + n, acc[i][j]);
						else tg_store4(g.C2 + (size_t)m * g.ldc2 + n - g.n_split, acc[i][j]);
					} else if constexpr (EPI == TG_GE_GELU) {
						f32x4_t r;
#pragma unroll
						for (int e = 0; e < 4; e++) r[e] = tg_gelu(acc[i][j][e]);
						tg_store4((T *)g.C + (size_t)m * g.ldc + n, r);
					} else if constexpr (EPI == TG_GE_F32) {
						tg_store4(g.C2 + (size_t)m * g.ldc2 + n, acc[i][j]);
					} else {
						float *c = g.C2 + (size_t)m * g.ldc2 + n;
						f32x4_t x = tg_load4(c);
#pragma unroll
						for (int e = 0; e < 4; e++) x[e] = x[e] + g.mult * acc[i][j][e];
						tg_store4(c, x);
					}
				}
			}
		}
	}
}

// Few columns (a router): 16 rows x 64 columns per workgroup, the waves share K, operands straight from memory in fragment
// order, partial sums meet in LDS.
template <class TR>
__global__ __launch_bounds__(256) void linear_thin_kernel(TgGemm g) {
	typedef typename TR::T T;
	typedef typename TR::Frag Frag;
	constexpr int NI = 4, U = 4;
	__shared__ f32x4_t s_acc[4][NI][64];
	const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, lr = lane & 15, lg = lane >> 4;
	const int m0 = blockIdx.x * 16, n0 = blockIdx.y * NI, kfr = g.K / TR::KF, nfr = g.N / 16;
	const T *A = (const T *)g.A + (size_t)min(m0 + lr, g.M - 1) * g.lda + lg * TR::KV;
	const Frag *W = reinterpret_cast<const Frag *>(g.W) + lane;
	f32x4_t acc[NI];
#pragma unroll
	for (int j = 0; j < NI; j++) acc[j] = f32x4_t{0, 0, 0, 0};
	for (int kf = w; kf < kfr; kf += 4 * U) {
		Frag a[U], b[U][NI];
#pragma unroll
		for (int u = 0; u < U; u++) {
			const int kc = min(kf + 4 * u, kfr - 1);
			a[u] = *reinterpret_cast<const Frag *>(A + (size_t)kc * TR::KF);
#pragma unroll
			for (int j = 0; j < NI; j++) b[u][j] = W[((size_t)min(n0 + j, nfr - 1) * kfr + kc) * 64];
		}
#pragma unroll
		for (int u = 0; u < U; u++) {
			if (kf + 4 * u >= kfr) a[u] = Frag{};
#pragma unroll
			for (int j = 0; j < NI; j++) acc[j] = TR::mma(b[u][j], a[u], acc[j]);
		}
	}
#pragma unroll
	for (int j = 0; j < NI; j++) s_acc[w][j][lane] = acc[j];
	__syncthreads();
	// wave w: column fragment w
	f32x4_t r;
#pragma unroll
	for (int e = 0; e < 4; e++) r[e] = (s_acc[0][w][lane][e] + s_acc[1][w][lane][e]) + (s_acc[2][w][lane][e] + s_acc[3][w][lane][e]);
	if (m0 + lr < g.M && n0 + w < nfr) tg_store4(g.C2 + (size_t)(m0 + lr) * g.ldc2 + (n0 + w) * 16 + 4 * lg, r);
}

template <class TR, int EPI>
void launch_linear_t(const TgGemm &g, hipStream_t s) {
	if constexpr (EPI == TG_GE_F32) {
		if (g.N <= 256) {
			hipLaunchKernelGGL((linear_thin_kernel<TR>), dim3((unsigned)((g.M + 15) / 16), (unsigned)((g.N + 63) / 64)), dim3(256), 0, s, g);
			return;
		}
	}
	if (g.tiles) {
		if constexpr (EPI == TG_GE_STORE || EPI == TG_GE_SWIGLU) {
			const unsigned grid = (unsigned)g.max_tiles * (unsigned)((g.N + 127) / 128);
			if (g.tile_rows == 128)
				hipLaunchKernelGGL((linear_kernel<TR, EPI, 2, 2, 4, 4, true>), dim3(grid), dim3(256), 0, s, g);
			else if (g.tile_rows == 64)
				hipLaunchKernelGGL((linear_kernel<TR, EPI, 2, 2, 2, 4, true>), dim3(grid), dim3(256), 0, s, g);
			else
				hipLaunchKernelGGL((linear_kernel<TR, EPI, 1, 4, 2, 2, true>), dim3(grid), dim3(256), 0, s, g);
		}
		return;
	}
	const int ntn = (g.N + 127) / 128, rows = EPI == TG_GE_TRANS ? g.rows_out : g.M;
	// 128-row tiles where they fill the device's 512 places (two workgroups per compute unit), then 64 rows, then 32
	const int t128 = (rows + 127) / 128 * ntn, t64 = (rows + 63) / 64 * ntn;
	if (t128 >= 448)
		hipLaunchKernelGGL((linear_kernel<TR, EPI, 2, 2, 4, 4, false>), dim3((unsigned)((rows + 127) / 128 * ntn)), dim3(256), 0, s, g);
	else if (t64 >= 256)
		hipLaunchKernelGGL((linear_kernel<TR, EPI, 2, 2, 2, 4, false>), dim3((unsigned)t64), dim3(256), 0, s, g);
	else
		hipLaunchKernelGGL((linear_kernel<TR, EPI, 1, 4, 2, 2, false>), dim3((unsigned)((rows + 31) / 32 * ntn)), dim3(256), 0, s, g);
}

template <class TR>
void launch_linear_dt(const TgGemm &g, int epi, hipStream_t s) {
	switch (epi) {
		case TG_GE_STORE: launch_linear_t<TR, TG_GE_STORE>(g, s); break;
		case TG_GE_F32: launch_linear_t<TR, TG_GE_F32>(g, s); break;
		case TG_GE_RESID: launch_linear_t<TR, TG_GE_RESID>(g, s); break;
		case TG_GE_GELU: launch_linear_t<TR, TG_GE_GELU>(g, s); break;
		case TG_GE_SWIGLU: launch_linear_t<TR, TG_GE_SWIGLU>(g, s); break;
		default: launch_linear_t<TR, TG_GE_TRANS>(g, s); break;
	}
}

unsigned pack_grid(const TgPack &p) {
	const long long n = ((long long)p.rows * p.cols + 255) / 256;
	return (unsigned)(n < 16384 ? (n > 0 ? n : 1) : 16384);
}

}  // namespace

void tg_launch_pack(const TgMat &dst, int dt, const TgPack &p, hipStream_t s) {
	if (dt == TG_DT_BF16) hipLaunchKernelGGL((pack_kernel<TgB16>), dim3(pack_grid(p)), dim3(256), 0, s, (__bf16 *)dst.w, dst.k, p);
	else hipLaunchKernelGGL((pack_kernel<TgF32>), dim3(pack_grid(p)), dim3(256), 0, s, (float *)dst.w, dst.k, p);
}

void tg_launch_unpack_f32(float *dst, int ld, const TgPack &p, hipStream_t s) {
	hipLaunchKernelGGL(unpack_f32_kernel, dim3(pack_grid(p)), dim3(256), 0, s, dst, ld, p);
}

int tg_vec_blocks(const TgVec &v, int epi) {
	if (vec_wide(v, epi)) return (v.ntiles + 3) / 4;
	return epi == TG_VE_SWIGLU || vec_pairs(v, epi) ? (v.ntiles + 1) / 2 : v.ntiles;
}

// Parts of K for a product whose consumer adds them: enough workgroups for the device, at least 8 fragments per part.
int tg_vec_ksplit(int ntiles, int nz, int kfrags, int n_cu) {
	int p = 1;
	while (p < 8 && ntiles * nz * p < n_cu && kfrags / (2 * p) >= 8) p *= 2;
	return p;
}

void tg_launch_vec(const TgVec &v, int dt, int pro, int epi, hipStream_t s) {
	if (dt == TG_DT_BF16) launch_vec_dt<TgB16>(v, pro, epi, s);
	else launch_vec_dt<TgF32>(v, pro, epi, s);
}

void tg_launch_linear(const TgGemm &g, int dt, int epi, hipStream_t s) {
	if (dt == TG_DT_BF16) launch_linear_dt<TgB16>(g, epi, s);
	else launch_linear_dt<TgF32>(g, epi, s);
}
