// Latent attention: tg_latent.h.

#include "tg_latent.h"

namespace {

// ---- one token -------------------------------------------------------------------------------------------------------------
// A workgroup takes one part of the keys for 16 heads and (blockIdx.z) 512 latent columns of the value sum.  Scores of a tile
// of 64 keys come from the matrix instructions (wave w: keys 16 w ...), the running softmax is a wave's work for 4 heads, the
// value sum stays on the vector units in fp32: a lane owns two latent columns of all 16 heads.
template <class TR>
__global__ __launch_bounds__(256) void latent_step_kernel(TgLatentStep a) {
	typedef typename TR::T T;
	typedef typename TR::Frag Frag;
	extern __shared__ __align__(16) unsigned char smem[];
	Frag *s_q = reinterpret_cast<Frag *>(smem);  // [rankp / KF][64]
	__shared__ __align__(16) float s_p[64][20];
	__shared__ float s_corr[16], s_sq[4];
	const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, lr = lane & 15, lg = lane >> 4;
	const int part = blockIdx.x, h0 = blockIdx.y * 16, heads16 = (int)gridDim.y * 16;
	const int pos = a.host_pos >= 0 ? a.host_pos : a.ctr[0], ctx = pos + 1;
	const int kb = part * a.chunk, ke = min(ctx, kb + a.chunk);
	T *cache = (T *)a.cache;

	// the new token's row, by the workgroup(s) whose part it ends
	if (pos >= kb && pos < kb + a.chunk) {
		float ss = 0.0f;
		for (int j = tid; j < a.rank; j += 256) ss = fmaf(a.dkv[j], a.dkv[j], ss);
		ss = tg_wave_sum(ss);
		if (lane == 0) s_sq[w] = ss;
		__syncthreads();
		const float inv = 1.0f / sqrtf(((s_sq[0] + s_sq[1]) + (s_sq[2] + s_sq[3])) / (float)a.rank + a.eps);
		for (int j = tid; j < a.rankp; j += 256) {
			const int jc = j < a.rank ? j : 0;
			const float c = a.dkv[jc] * inv * a.norm[jc];
			cache[(size_t)pos * a.rankp + j] = (T)(j < a.rank ? c : 0.0f);
		}
	}
	// q' in operand order: lane = head, 16 bytes of the latent
	for (int e = tid; e < 16 * a.rankp; e += 256) {
		const int h = e / a.rankp, j = e - h * a.rankp, hh = h0 + h;
		const float v = hh < a.heads ? a.q[(size_t)hh * a.rankp + j] : 0.0f;
		reinterpret_cast<T *>(s_q)[((size_t)(j / TR::KF) * 64 + h + 16 * ((j % TR::KF) / TR::KV)) * TR::KV + j % TR::KV] = (T)v;
	}
	__syncthreads();

	const int col = blockIdx.z * 512 + 2 * tid;
	const bool cin = col < a.rankp;
	const int colc = cin ? col : 0;
	float acc[16][2];
#pragma unroll
	for (int h = 0; h < 16; h++) acc[h][0] = acc[h][1] = 0.0f;
	float m[4], l[4];
#pragma unroll
	for (int i = 0; i < 4; i++) { m[i] = -INFINITY; l[i] = 0.0f; }
	const int kfr = a.rankp / TR::KF;
	for (int k0 = kb; k0 < ke; k0 += 64) {
		{
			const int key = min(k0 + 16 * w + lr, ke - 1);
			const T *row = cache + (size_t)key * a.rankp + lg * TR::KV;
			f32x4_t sc = {0, 0, 0, 0};
			for (int kf = 0; kf < kfr; kf++) sc = TR::mma(*reinterpret_cast<const Frag *>(row + (size_t)kf * TR::KF), s_q[kf * 64 + lane], sc);
#pragma unroll
			for (int e = 0; e < 4; e++) s_p[16 * w + 4 * lg + e][lr] = k0 + 16 * w + 4 * lg + e < ke ? sc[e] * a.scale : -INFINITY;
		}
		__syncthreads();
#pragma unroll
		for (int i = 0; i < 4; i++) {
			const float s = s_p[lane][4 * w + i];
			const float mn = fmaxf(m[i], tg_wave_max(s)), f = expf(m[i] - mn), p = expf(s - mn);
			s_p[lane][4 * w + i] = p;
			l[i] = l[i] * f + tg_wave_sum(p);
			m[i] = mn;
			if (lane == 0) s_corr[4 * w + i] = f;
		}
		__syncthreads();
#pragma unroll
		for (int h = 0; h < 16; h++) {
			acc[h][0] *= s_corr[h];
			acc[h][1] *= s_corr[h];
		}
		const int kn = min(64, ke - k0);
		const T *base = cache + (size_t)k0 * a.rankp + colc;
		for (int k = 0; k < kn; k += 8) {
			float c0[8], c1[8];
#pragma unroll
			for (int u = 0; u < 8; u++) {
				const T *p = base + (size_t)min(k + u, kn - 1) * a.rankp;
				c0[u] = (float)p[0];
				c1[u] = (float)p[1];
			}
#pragma unroll
			for (int u = 0; u < 8; u++) {  // rows past the part's end have probability 0
				const int kk = k + u;
#pragma unroll
				for (int h4 = 0; h4 < 4; h4++) {
					const f32x4_t p = tg_load4(&s_p[kk][4 * h4]);
#pragma unroll
					for (int e = 0; e < 4; e++) {
						acc[4 * h4 + e][0] = fmaf(p[e], c0[u], acc[4 * h4 + e][0]);
						acc[4 * h4 + e][1] = fmaf(p[e], c1[u], acc[4 * h4 + e][1]);
					}
				}
			}
		}
		__syncthreads();
	}
	if (cin) {
		float *o = a.part_acc + ((size_t)part * heads16 + h0) * a.rankp + col;
#pragma unroll
		for (int h = 0; h < 16; h++) *reinterpret_cast<float2 *>(o + (size_t)h * a.rankp) = float2{acc[h][0], acc[h][1]};
	}
	if (blockIdx.z == 0 && lane == 0) {
#pragma unroll
		for (int i = 0; i < 4; i++) {
			float *ml = a.part_ml + ((size_t)part * heads16 + h0 + 4 * w + i) * 2;
			ml[0] = m[i];
			ml[1] = l[i];
		}
	}
}

__global__ __launch_bounds__(256) void latent_fold_kernel(const float *acc, const float *ml, int nb, int heads16, int rankp, float *out_acc,
                                                          float *out_ml) {
	__shared__ float s_f[TG_LATENT_MAX_BLOCKS];
	__shared__ float s_r[4];
	const int h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
	float m = -INFINITY;
	for (int b = tid; b < nb; b += 256) m = fmaxf(m, ml[((size_t)b * heads16 + h) * 2]);
	m = tg_wave_max(m);
	if (lane == 0) s_r[w] = m;
	__syncthreads();
	m = fmaxf(fmaxf(s_r[0], s_r[1]), fmaxf(s_r[2], s_r[3]));
	__syncthreads();
	float l = 0.0f;
	for (int b = tid; b < nb; b += 256) {
		const float f = expf(ml[((size_t)b * heads16 + h) * 2] - m);
		s_f[b] = f;
		l += f * ml[((size_t)b * heads16 + h) * 2 + 1];
	}
	l = tg_wave_sum(l);
	if (lane == 0) s_r[w] = l;
	__syncthreads();
	if (tid == 0 && blockIdx.y == 0) {
		out_ml[2 * h] = m;
		out_ml[2 * h + 1] = (s_r[0] + s_r[1]) + (s_r[2] + s_r[3]);
	}
	const int j = blockIdx.y * 64 + lane;  // a wave per quarter of the parts
	float a = 0.0f;
	for (int b = w; b < nb; b += 4) a = fmaf(s_f[b], acc[((size_t)b * heads16 + h) * rankp + j], a);
	__shared__ float s_a[4][64];
	s_a[w][lane] = a;
	__syncthreads();
	if (w == 0) out_acc[(size_t)h * rankp + j] = (s_a[0][lane] + s_a[1][lane]) + (s_a[2][lane] + s_a[3][lane]);
}

// ---- many tokens -------------------------------------------------------------------------------------------------------------
template <class TR>
__global__ __launch_bounds__(256) void latent_rows_kernel(const float *dkv, int ld, int n, int rank, int rankp, const float *norm, float eps,
                                                          typename TR::T *rows) {
	const int t = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
	if (t >= n) return;
	const float *x = dkv + (size_t)t * ld;
	float ss = 0.0f;
	for (int j = lane; j < rank; j += 64) ss = fmaf(x[j], x[j], ss);
	ss = tg_wave_sum(ss);
	const float inv = 1.0f / sqrtf(ss / (float)rank + eps);
	for (int j = lane; j < rankp; j += 64) {
		const int jc = j < rank ? j : 0;
		const float c = x[jc] * inv * norm[jc];
		rows[(size_t)t * rankp + j] = (typename TR::T)(j < rank ? c : 0.0f);
	}
}

// A workgroup: one head, 64 QT queries (wave: 16 QT of them).  Per tile of KT keys: K and V^T fragments go global ->
// registers -> LDS, the next tile's loads in flight during this one's arithmetic.  Scores are taken as K Q^T, so a lane holds
// four consecutive keys of one query and the probabilities are already the second operand of V^T P^T; in the bf16 format they
// enter it as two bf16 planes (value and remainder).
template <class TR, int DMAX, int KT, int QT>
__global__ __launch_bounds__(256) void latent_attn_kernel(TgLatentRows a) {
	typedef typename TR::T T;
	typedef typename TR::Frag Frag;
	constexpr int ND = DMAX / TR::KF, NV = DMAX / 16, NK = KT / 16, NB = KT / TR::KF;
	constexpr int KFRAGS = NK * ND, NF = KFRAGS + NV * NB, PW = NF / 4;
	static_assert(NF % 4 == 0 && NB >= 1, "");
	__shared__ __align__(16) Frag lds[NF * 64];
	const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, lr = lane & 15, lg = lane >> 4;
	const int h = blockIdx.x, qb = ((int)gridDim.y - 1 - (int)blockIdx.y) * 64 * QT;  // the longest rows first
	const int kd = a.dimp / TR::KF, nv = a.vdimp / 16;
	const T *Q = (const T *)a.q, *K = (const T *)a.k + (size_t)h * a.dimp, *V = (const T *)a.vt + (size_t)h * a.vdimp * a.ldv;
	const float sl2 = a.scale * 1.44269504088896340736f;

	Frag qf[QT][ND];
	int qi[QT];
#pragma unroll
	for (int s = 0; s < QT; s++) {
		qi[s] = qb + w * 16 * QT + s * 16 + lr;
		const T *row = Q + (size_t)min(qi[s], a.n - 1) * a.ldq + (size_t)h * a.dimp + lg * TR::KV;
#pragma unroll
		for (int d = 0; d < ND; d++) qf[s][d] = *reinterpret_cast<const Frag *>(row + (d < kd ? d : 0) * TR::KF);
	}
	f32x4_t o[QT][NV];
	float m[QT], l[QT];
#pragma unroll
	for (int s = 0; s < QT; s++) {
		m[s] = -INFINITY;
		l[s] = 0.0f;
#pragma unroll
		for (int v = 0; v < NV; v++) o[s][v] = f32x4_t{0, 0, 0, 0};
	}
	const int last = a.past + min(qb + 64 * QT, a.n) - 1;  // the last key any of these queries sees
	const int nt = last / KT + 1, ctx = a.past + a.n;
	Frag st[PW];
	auto fetch = [&](int k0) {
#pragma unroll
		for (int i = 0; i < PW; i++) {
			const int f = i * 4 + w;
			const T *p;
			if (f < KFRAGS) {
				const int kt = f / ND, d = f % ND;
				p = K + (size_t)min(k0 + kt * 16 + lr, ctx - 1) * a.ldk + (d < kd ? d : 0) * TR::KF + lg * TR::KV;
			} else {
				const int v = (f - KFRAGS) / NB, b = (f - KFRAGS) % NB;
				p = V + (size_t)((v < nv ? v : 0) * 16 + lr) * a.ldv + k0 + b * TR::KF + lg * TR::KV;
			}
			st[i] = *reinterpret_cast<const Frag *>(p);
		}
	};
	auto put = [&]() {
#pragma unroll
		for (int i = 0; i < PW; i++) lds[(i * 4 + w) * 64 + lane] = st[i];
	};
	fetch(0);
	put();
	tg_lds_barrier();
	for (int t = 0; t < nt; t++) {
		const int k0 = t * KT;
		fetch((t + 1 < nt ? t + 1 : t) * KT);
		f32x4_t sc[QT][NK];
#pragma unroll
		for (int kt = 0; kt < NK; kt++) {
#pragma unroll
			for (int s = 0; s < QT; s++) sc[s][kt] = f32x4_t{0, 0, 0, 0};
#pragma unroll
			for (int d = 0; d < ND; d++)
				if (d < kd) {
					const Frag kf = lds[(kt * ND + d) * 64 + lane];
#pragma unroll
					for (int s = 0; s < QT; s++) sc[s][kt] = TR::mma(kf, qf[s][d], sc[s][kt]);
				}
		}
#pragma unroll
		for (int s = 0; s < QT; s++) {
			const int lim = a.past + qi[s];
			float mt = -INFINITY;
#pragma unroll
			for (int kt = 0; kt < NK; kt++)
#pragma unroll
				for (int e = 0; e < 4; e++) {
					const float v = k0 + kt * 16 + 4 * lg + e <= lim ? sc[s][kt][e] * sl2 : -INFINITY;
					sc[s][kt][e] = v;
					mt = fmaxf(mt, v);
				}
			mt = fmaxf(mt, tg_red_partner<32>(mt));
			mt = fmaxf(mt, tg_red_partner<16>(mt));
			const float mn = fmaxf(m[s], mt), f = exp2f(m[s] - mn);  // key 0 is in the first tile: mn is finite
			m[s] = mn;
			float sum = 0.0f;
#pragma unroll
			for (int kt = 0; kt < NK; kt++)
#pragma unroll
				for (int e = 0; e < 4; e++) {
					const float p = exp2f(sc[s][kt][e] - mn);
					sc[s][kt][e] = p;
					sum += p;
				}
			l[s] = l[s] * f + sum;
#pragma unroll
			for (int v = 0; v < NV; v++)
#pragma unroll
				for (int e = 0; e < 4; e++) o[s][v][e] *= f;
		}
#pragma unroll
		for (int b = 0; b < NB; b++) {
			Frag ph[QT], pl[QT];
#pragma unroll
			for (int s = 0; s < QT; s++) {
				if constexpr (TR::DT == TG_DT_BF16) {
#pragma unroll
					for (int e = 0; e < 8; e++) {
						const float p = sc[s][2 * b + (e >> 2)][e & 3];
						const __bf16 hi = (__bf16)p;
						ph[s][e] = hi;
						pl[s][e] = (__bf16)(p - (float)hi);
					}
				} else {
					ph[s] = sc[s][b];
				}
			}
#pragma unroll
			for (int v = 0; v < NV; v++)
				if (v < nv) {
					const Frag vf = lds[(KFRAGS + v * NB + b) * 64 + lane];
#pragma unroll
					for (int s = 0; s < QT; s++) {
						o[s][v] = TR::mma(vf, ph[s], o[s][v]);
						if constexpr (TR::DT == TG_DT_BF16) o[s][v] = TR::mma(vf, pl[s], o[s][v]);
					}
				}
		}
		tg_lds_barrier();
		put();
		tg_lds_barrier();
	}
#pragma unroll
	for (int s = 0; s < QT; s++) {
		float ls = l[s];
		ls += tg_red_partner<32>(ls);
		ls += tg_red_partner<16>(ls);
		if (qi[s] >= a.n) continue;
		const float f = tg_sigmoid(a.gate[(size_t)qi[s] * a.ld_gate + h]) / ls;
		T *dst = (T *)a.out + (size_t)qi[s] * a.ldo + (size_t)h * a.vdimp + 4 * lg;
#pragma unroll
		for (int v = 0; v < NV; v++)
			if (v < nv) {
				f32x4_t r;
#pragma unroll
				for (int e = 0; e < 4; e++) r[e] = o[s][v][e] * f;
				tg_store4(dst + v * 16, r);
			}
		if (h == a.heads - 1)
			for (int c = a.heads * a.vdimp + 4 * lg; c < a.ldo; c += 16) tg_store4((T *)a.out + (size_t)qi[s] * a.ldo + c, f32x4_t{0, 0, 0, 0});
	}
}

template <class TR>
void launch_attention(const TgLatentRows &a, hipStream_t s) {
	const int d = a.dimp > a.vdimp ? a.dimp : a.vdimp;
	const dim3 g1((unsigned)a.heads, (unsigned)((a.n + 63) / 64)), g2((unsigned)a.heads, (unsigned)((a.n + 127) / 128));
	const bool two = TR::DT == TG_DT_BF16 && a.heads * ((a.n + 127) / 128) >= 512;  // 128-query tiles where they fill the device twice
	if (d <= 64) {
		if (two) hipLaunchKernelGGL((latent_attn_kernel<TR, 64, 64, 2>), g2, dim3(256), 0, s, a);
		else hipLaunchKernelGGL((latent_attn_kernel<TR, 64, 64, 1>), g1, dim3(256), 0, s, a);
	} else if (d <= 128) {
		if (two) hipLaunchKernelGGL((latent_attn_kernel<TR, 128, 64, 2>), g2, dim3(256), 0, s, a);
		else hipLaunchKernelGGL((latent_attn_kernel<TR, 128, 64, 1>), g1, dim3(256), 0, s, a);
	} else {
		hipLaunchKernelGGL((latent_attn_kernel<TR, 256, 32, 1>), g1, dim3(256), 0, s, a);
	}
}

}  // namespace

void tg_launch_latent_step(const TgLatentStep &a, int dt, hipStream_t s) {
	const dim3 grid((unsigned)a.nb, (unsigned)((a.heads + 15) / 16), (unsigned)((a.rankp + 511) / 512));
	const size_t lds = 16 * (size_t)a.rankp * tg_dt_bytes(dt);
	if (dt == TG_DT_BF16) hipLaunchKernelGGL((latent_step_kernel<TgB16>), grid, dim3(256), lds, s, a);
	else hipLaunchKernelGGL((latent_step_kernel<TgF32>), grid, dim3(256), lds, s, a);
}

void tg_launch_latent_fold(const float *acc, const float *ml, int nb, int heads16, int rankp, float *out_acc, float *out_ml, hipStream_t s) {
	hipLaunchKernelGGL(latent_fold_kernel, dim3((unsigned)heads16, (unsigned)(rankp / 64)), dim3(256), 0, s, acc, ml, nb, heads16, rankp, out_acc,
	                   out_ml);
}

void tg_launch_latent_rows(const float *dkv, int ld, int n, int rank, int rankp, const float *norm, float eps, int dt, void *cache_rows,
                           hipStream_t s) {
	const dim3 grid((unsigned)((n + 3) / 4));
	if (dt == TG_DT_BF16)
		hipLaunchKernelGGL((latent_rows_kernel<TgB16>), grid, dim3(256), 0, s, dkv, ld, n, rank, rankp, norm, eps, (__bf16 *)cache_rows);
	else
		hipLaunchKernelGGL((latent_rows_kernel<TgF32>), grid, dim3(256), 0, s, dkv, ld, n, rank, rankp, norm, eps, (float *)cache_rows);
}

void tg_launch_latent_attention(const TgLatentRows &a, int dt, hipStream_t s) {
	if (dt == TG_DT_BF16) launch_attention<TgB16>(a, s);
	else launch_attention<TgF32>(a, s);
}
