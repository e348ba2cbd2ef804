// Latent attention: tg_latent.h.

#include "tg_latent.h"

namespace {

// ---- one token -------------------------------------------------------------------------------------------------------------
// A workgroup takes one part of the keys for 16 heads, tile by tile of 32.  A tile's latent rows go to LDS in one round trip
// (the first tile's loads are requested before anything else is done), row pitch 16 bytes more than the row.  Scores: wave w
// takes keys 16 (w % 2) ... and half w / 2 of the latent; the running softmax is a wave's work for 4 heads; the value sum is
// a product of the probabilities [16 heads x 32 keys] (in the bf16 format two planes, value and remainder) with the tile,
// wave w the column tiles w, w + 4, ..., NC of them; wider rows take several workgroups (blockIdx.z).
constexpr int ST = 32;         // keys per tile
template <bool ROT>
constexpr int ST_LOADS = ROT ? 10 : 8;  // 16-byte pieces per lane and round of the tile copy

template <class TR>
size_t latent_step_lds(int rowp) {  // q' fragments | tile
	const size_t row = (size_t)rowp * sizeof(typename TR::T);
	return 16 * row + ST * (row + 16);
}

// Element i of a rotated vector: itself, turned with its partner.
struct Turn {
	int other, pair;
	bool turns, second;
	__device__ __forceinline__ Turn(int i, int dims, int half_layout) {
		const int hd = dims / 2;
		turns = i < dims;
		second = half_layout ? i >= hd : (i & 1) != 0;
		pair = !turns ? 0 : (half_layout ? (second ? i - hd : i) : i >> 1);
		other = !turns ? i : (half_layout ? (second ? i - hd : i + hd) : i ^ 1);
	}
	__device__ __forceinline__ float operator()(float v, float o, float2 t) const {
		return turns ? fmaf(v, t.x, second ? o * t.y : -(o * t.y)) : v;
	}
};
template <class V>
__device__ __forceinline__ float rotated(const V *x, int i, const float2 *turn, int dims, int half_layout) {
	const Turn r(i, dims, half_layout);
	return r((float)x[i], (float)x[r.other], turn[r.pair]);
}
// e / d for e * d < 2^22, m = 2^22 / d rounded up
__device__ __forceinline__ int div_by(int e, unsigned m) { return (int)(((unsigned)e * m) >> 22); }

// NC: column tiles of the value part per wave (4 NC tiles of 16 per workgroup).
template <class TR, bool ROT, int NC>
__global__ __launch_bounds__(256) void latent_step_kernel(TgLatentStep a) {
	typedef typename TR::T T;
	typedef typename TR::Frag Frag;
	extern __shared__ __align__(16) unsigned char smem[];
	const int rowp = a.rankp + (ROT ? a.rotp : 0), row = rowp * (int)sizeof(T), pitch = row + 16, ppr = row / 16;  // bytes; 16-byte pieces per row
	Frag *s_q = reinterpret_cast<Frag *>(smem);  // [rowp / KF][64]
	unsigned char *s_c = smem + 16 * row;
	__shared__ float s_half[2][ST][16];
	__shared__ __align__(16) float s_p[16][ST + 4];
	__shared__ float s_corr[16], s_sq[4];
	const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, lr = lane & 15, lg = lane >> 4;
	const int blocks = (a.heads + 15) / 16, grp = (int)blockIdx.y / blocks, hb = (int)blockIdx.y - grp * blocks;
	const int part = blockIdx.x, h0 = hb * 16, heads16 = (int)gridDim.y * 16, g0 = grp * a.heads;  // (h0: inside the group)
	const int pos = a.host_pos >= 0 ? a.host_pos : a.ctr[0], ctx = pos + 1, lo = max(0, ctx - a.window);
	const int kb = lo + part * a.chunk, ke = min(ctx, kb + a.chunk);
	const size_t key_bytes = (size_t)a.groups * row;
	unsigned char *cache = (unsigned char *)a.cache + (size_t)grp * row;
	const float2 *turn = ROT ? a.rot.table + (size_t)pos * (a.rot.dims / 2) : nullptr;
	constexpr int SL = ST_LOADS<ROT>;
	const unsigned mppr = ((1u << 22) + (unsigned)ppr - 1) / (unsigned)ppr;  // (32 ppr^2 < 2^22: rows below 5 KiB)
	typedef unsigned u32x4 __attribute__((ext_vector_type(4)));
	u32x4 piece[SL];
	// pieces [base, base + 256 * SL) of a tile; the new token's row is not in memory yet: it is written to LDS below
	auto request = [&](int k0, int base) {
#pragma unroll
		for (int i = 0; i < SL; i++) {
			const int e = min(base + tid + 256 * i, ST * ppr - 1), r = div_by(e, mppr), key = max(min(min(k0 + r, ke - 1), pos - 1), 0);
			piece[i] = *reinterpret_cast<const u32x4 *>(cache + (size_t)key * key_bytes + (e - r * ppr) * 16);
		}
	};
	auto place = [&](int base) {
#pragma unroll
		for (int i = 0; i < SL; i++) {
			const int e = base + tid + 256 * i, r = div_by(e, mppr);
			if (e < ST * ppr) *reinterpret_cast<u32x4 *>(s_c + (size_t)r * pitch + (e - r * ppr) * 16) = piece[i];
		}
	};
	const bool mine = pos >= kb && pos < kb + a.chunk;
	const float *kv = a.kv + (size_t)grp * a.kv_stride;
	float raw[2], nrm[2];
#pragma unroll
	for (int i = 0; i < 2; i++) {
		const int j = min(tid + 256 * i, a.rank - 1);
		raw[i] = kv[j];
		nrm[i] = a.norm ? a.norm[j] : 1.0f;
	}
	// rotated parts: of the queries (16 * rotp elements, RB of them per lane and pass) and of the new row
	constexpr int RB = 4;
	float rx[RB], ro[RB], kx = 0.0f, ko = 0.0f;
	float2 rt[RB], kt = {0.0f, 0.0f};
	unsigned mrot = 0;
	auto rot_request = [&](int base) {
#pragma unroll
		for (int i = 0; i < RB; i++) {
			const int e = min(base + tid + 256 * i, 16 * a.rotp - 1), h = div_by(e, mrot), j = min(e - h * a.rotp, a.rot_size - 1);
			const Turn r(j, a.rot.dims, a.rot.half_layout);
			const float *x = a.qr + (size_t)(g0 + min(h0 + h, a.heads - 1)) * a.qr_stride;
			rx[i] = x[j];
			ro[i] = x[r.other];
			rt[i] = turn[r.pair];
		}
	};
	auto rot_place = [&](int base) {
#pragma unroll
		for (int i = 0; i < RB; i++) {
			const int e = base + tid + 256 * i, h = div_by(min(e, 16 * a.rotp - 1), mrot), j = e - h * a.rotp, c = a.rankp + j;
			const Turn r(j, a.rot.dims, a.rot.half_layout);
			const float v = j < a.rot_size && h0 + h < a.heads ? r(rx[i], ro[i], rt[i]) : 0.0f;
			if (e < 16 * a.rotp)
				reinterpret_cast<T *>(s_q)[((size_t)(c / TR::KF) * 64 + h + 16 * ((c % TR::KF) / TR::KV)) * TR::KV + c % TR::KV] = (T)v;
		}
	};
	if constexpr (ROT) {
		mrot = ((1u << 22) + (unsigned)a.rotp - 1) / (unsigned)a.rotp;
		const int j = min(tid, a.rot_size - 1);
		const Turn r(j, a.rot.dims, a.rot.half_layout);
		const float *x = a.kr + (size_t)grp * a.kr_stride;
		kx = x[j];
		ko = x[r.other];
		kt = turn[r.pair];
		rot_request(0);
	}
	request(kb, 0);

	// q' in operand order: lane = head, 16 bytes of the row
	const int r4 = a.rankp / 4;
	const unsigned mr4 = ((1u << 22) + (unsigned)r4 - 1) / (unsigned)r4;
	for (int base = 0; base < 16 * r4; base += 256 * 8) {
		f32x4_t v[8];
#pragma unroll
		for (int i = 0; i < 8; i++) {
			const int e = min(base + tid + 256 * i, 16 * r4 - 1), h = div_by(e, mr4);
			v[i] = tg_load4(a.q + (size_t)(g0 + min(h0 + h, a.heads - 1)) * a.q_stride + (e - h * r4) * 4);
		}
#pragma unroll
		for (int i = 0; i < 8; i++) {
			const int e = base + tid + 256 * i, h = div_by(min(e, 16 * r4 - 1), mr4), j = (e - h * r4) * 4;
			if (h0 + h >= a.heads) v[i] = f32x4_t{0, 0, 0, 0};
			if constexpr (ROT) {
#pragma unroll
				for (int c = 0; c < 4; c++)
					if (j + c < a.q_zero) v[i][c] = 0.0f;
			}
			if (e < 16 * r4)
				tg_store4(reinterpret_cast<T *>(s_q) + ((size_t)(j / TR::KF) * 64 + h + 16 * ((j % TR::KF) / TR::KV)) * TR::KV + j % TR::KV, v[i]);
		}
	}
	if constexpr (ROT) {
		rot_place(0);
		for (int base = 256 * RB; base < 16 * a.rotp; base += 256 * RB) {
			rot_request(base);
			rot_place(base);
		}
	}
	// the new token's latent, normalised, by the workgroups whose part it ends
	float inv = 1.0f;
	if (mine && a.norm) {
		float ss = 0.0f;
		for (int j = tid, i = 0; j < a.rank; j += 256, i++) {
			const float x = i < 2 ? raw[i & 1] : kv[j];
			ss = fmaf(x, x, ss);
		}
		ss = tg_wave_sum(ss);
		if (lane == 0) s_sq[w] = ss;
		__syncthreads();
		inv = 1.0f / sqrtf(((s_sq[0] + s_sq[1]) + (s_sq[2] + s_sq[3])) / (float)a.rank + a.eps);
	}

	const int ct0 = blockIdx.z * (4 * NC) + w, nct = a.rankp / 16;
	f32x4_t acc[NC];
#pragma unroll
	for (int c = 0; c < NC; c++) acc[c] = f32x4_t{0, 0, 0, 0};
	float m[2], l[2];
#pragma unroll
	for (int i = 0; i < 2; i++) { m[i] = -INFINITY; l[i] = 0.0f; }
	const int kfr = rowp / TR::KF, kh = (kfr + 1) / 2, kf_lo = (w >> 1) * kh, kf_hi = min(kfr, kf_lo + kh);
	for (int k0 = kb; k0 < ke; k0 += ST) {
		for (int base = 0; base < ST * ppr; base += 256 * SL) {
			if (base) request(k0, base);
			place(base);
		}
		__syncthreads();
		if (mine && pos < k0 + ST) {
			T *dst = reinterpret_cast<T *>(cache + (size_t)pos * key_bytes), *tile = reinterpret_cast<T *>(s_c + (size_t)(pos - k0) * pitch);
			for (int j = tid, i = 0; j < a.rankp; j += 256, i++) {
				const int jc = j < a.rank ? j : 0;
				const float x = i < 2 ? raw[i & 1] : kv[jc], g = i < 2 ? nrm[i & 1] : (a.norm ? a.norm[jc] : 1.0f);
				const T c = (T)(j < a.rank ? x * inv * g : 0.0f);
				tile[j] = c;
				dst[j] = c;
			}
			if constexpr (ROT) {
				if (tid < a.rotp) {  // (rotp is at most 256)
					const Turn r(tid, a.rot.dims, a.rot.half_layout);
					const T c = (T)(tid < a.rot_size ? r(kx, ko, kt) : 0.0f);
					tile[a.rankp + tid] = c;
					dst[a.rankp + tid] = c;
				}
			}
			__syncthreads();
		}
		if (k0 + ST < ke) request(k0 + ST, 0);
		{
			const unsigned char *rp = s_c + (size_t)(16 * (w & 1) + lr) * pitch + lg * 16;
			f32x4_t sc = {0, 0, 0, 0};
			for (int kf = kf_lo; kf < kf_hi; kf++) sc = TR::mma(*reinterpret_cast<const Frag *>(rp + kf * 64), s_q[kf * 64 + lane], sc);
#pragma unroll
			for (int e = 0; e < 4; e++) s_half[w >> 1][16 * (w & 1) + 4 * lg + e][lr] = sc[e];
		}
		__syncthreads();
		{
			// lane: key lane % 32, heads 4 w + lane / 32 and 4 w + 2 + lane / 32
			const int key = lane & 31;
#pragma unroll
			for (int i = 0; i < 2; i++) {
				const int h = 4 * w + 2 * i + (lane >> 5);
				const float s = k0 + key < ke ? (s_half[0][key][h] + s_half[1][key][h]) * a.scale : -INFINITY;
				float mx = fmaxf(s, tg_red_partner<16>(s));
				mx = tg_row16_max(mx);
				const float mn = fmaxf(m[i], mx), f = expf(m[i] - mn), p = expf(s - mn);
				float sum = p + tg_red_partner<16>(p);
				sum = tg_row16_sum(sum);
				s_p[h][key] = p;
				l[i] = l[i] * f + sum;
				m[i] = mn;
				if (key == 0) s_corr[h] = f;
			}
		}
		__syncthreads();
		if (k0 > kb) {
#pragma unroll
			for (int e = 0; e < 4; e++) {
				const float f = s_corr[4 * lg + e];
#pragma unroll
				for (int c = 0; c < NC; c++) acc[c][e] *= f;
			}
		}
		// rows past the part's end repeat its last row, with probability 0
#pragma unroll
		for (int b = 0; b < ST / TR::KF; b++) {
			Frag ph, pl;
			f32x4_t pv[TR::KV / 4];
#pragma unroll
			for (int i = 0; i < TR::KV / 4; i++) pv[i] = tg_load4(&s_p[lr][b * TR::KF + lg * TR::KV + 4 * i]);
#pragma unroll
			for (int i = 0; i < TR::KV; i++) {
				const T hi = (T)pv[i / 4][i % 4];
				ph[i] = hi;
				pl[i] = (T)(pv[i / 4][i % 4] - (float)hi);
			}
#pragma unroll
			for (int c = 0; c < NC; c++) {
				const int ct = min(ct0 + 4 * c, nct - 1);
				const T *col = reinterpret_cast<const T *>(s_c + (size_t)(b * TR::KF + lg * TR::KV) * pitch) + ct * 16 + lr;
				Frag cf;
#pragma unroll
				for (int i = 0; i < TR::KV; i++) cf[i] = *reinterpret_cast<const T *>(reinterpret_cast<const unsigned char *>(col) + i * pitch);
				acc[c] = TR::mma(ph, cf, acc[c]);
				if constexpr (TR::DT == TG_DT_BF16) acc[c] = TR::mma(pl, cf, acc[c]);
			}
		}
		__syncthreads();
	}
	const int hp = (int)blockIdx.y * 16;  // this block's padded heads
	float *o = a.part_acc + ((size_t)part * heads16 + hp) * a.rankp;
#pragma unroll
	for (int c = 0; c < NC; c++) {
		const int ct = ct0 + 4 * c;
		if (ct < nct) {
#pragma unroll
			for (int e = 0; e < 4; e++) o[(size_t)(4 * lg + e) * a.rankp + ct * 16 + lr] = acc[c][e];
		}
	}
	if (blockIdx.z == 0 && (lane & 31) == 0) {
#pragma unroll
		for (int i = 0; i < 2; i++) {
			float *ml = a.part_ml + ((size_t)part * heads16 + hp + 4 * w + 2 * i + (lane >> 5)) * 2;
			ml[0] = m[i];
			ml[1] = l[i];
		}
	}
}

// groups > 0: the normalised sum of real head (group, head) instead, [groups * heads][out_stride]
__global__ __launch_bounds__(256) void latent_fold_kernel(const float *acc, const float *ml, int nb, int heads16, int rankp, float *out_acc,
                                                          float *out_ml, int groups, int heads, int out_stride) {
	__shared__ float s_f[TG_LATENT_MAX_BLOCKS];
	__shared__ float s_r[4];
	const int hp16 = (heads + 15) / 16 * 16, real = (int)blockIdx.x;
	const int h = groups ? real / heads * hp16 + real % heads : real, tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
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
	l = (s_r[0] + s_r[1]) + (s_r[2] + s_r[3]);
	if (!groups && tid == 0 && blockIdx.y == 0) {
		out_ml[2 * h] = m;
		out_ml[2 * h + 1] = l;
	}
	const int j = blockIdx.y * 64 + lane, jc = min(j, rankp - 1);  // a wave per quarter of the parts
	float a = 0.0f;
	for (int b = w; b < nb; b += 64) {
		float v[16];
#pragma unroll
		for (int i = 0; i < 16; i++) v[i] = acc[((size_t)min(b + 4 * i, nb - 1) * heads16 + h) * rankp + jc];
#pragma unroll
		for (int i = 0; i < 16; i++) a = fmaf(b + 4 * i < nb ? s_f[min(b + 4 * i, nb - 1)] : 0.0f, v[i], a);
	}
	__shared__ float s_a[4][64];
	s_a[w][lane] = a;
	__syncthreads();
	if (w != 0 || j >= rankp) return;
	const float sum = (s_a[0][lane] + s_a[1][lane]) + (s_a[2][lane] + s_a[3][lane]);
	if (groups) out_acc[(size_t)real * out_stride + j] = sum / l;
	else out_acc[(size_t)h * rankp + j] = sum;
}

// ---- many tokens -------------------------------------------------------------------------------------------------------------
// a wave per token and group
template <class TR, class SRC>
__global__ __launch_bounds__(256) void latent_rows_kernel(TgLatentCacheRows a) {
	typedef typename TR::T T;
	const int e = blockIdx.x * 4 + (threadIdx.x >> 6), t = e / a.groups, grp = e - t * a.groups, lane = threadIdx.x & 63;
	if (t >= a.n) return;
	const SRC *x = (const SRC *)a.kv + (size_t)t * a.ld + (size_t)grp * a.kv_stride, *r = (const SRC *)a.kr + (size_t)t * a.ld + (size_t)grp * a.kr_stride;
	float inv = 1.0f;
	if (a.norm) {
		float ss = 0.0f;
		for (int j = lane; j < a.rank; j += 64) ss = fmaf((float)x[j], (float)x[j], ss);
		ss = tg_wave_sum(ss);
		inv = 1.0f / sqrtf(ss / (float)a.rank + a.eps);
	}
	const int pos = a.past + t;
	T *row = (T *)a.cache + ((size_t)pos * a.groups + grp) * (a.rankp + a.rotp);
	for (int j = lane; j < a.rankp; j += 64) {
		const int jc = j < a.rank ? j : 0;
		const float c = (float)x[jc] * inv * (a.norm ? a.norm[jc] : 1.0f);
		row[j] = (T)(j < a.rank ? c : 0.0f);
	}
	const float2 *turn = a.rot.table + (size_t)pos * (a.rot.dims / 2);
	for (int j = lane; j < a.rotp; j += 64) row[a.rankp + j] = (T)(j < a.rot_size ? rotated(r, j, turn, a.rot.dims, a.rot.half_layout) : 0.0f);
}

// a lane per pair
template <class T>
__global__ __launch_bounds__(256) void rot_rows_kernel(T *rows, int ld, int past, int first, int count, int stride, TgRot rot) {
	const int hd = rot.dims / 2, per = count * hd, t = blockIdx.y;
	const int e = blockIdx.x * 256 + threadIdx.x;
	if (e >= per) return;
	const int v = e / hd, i = e - v * hd;
	T *x = rows + (size_t)t * ld + first + (size_t)v * stride;
	T *p = x + (rot.half_layout ? i : 2 * i), *q = x + (rot.half_layout ? i + hd : 2 * i + 1);
	const float2 c = rot.table[(size_t)(past + t) * hd + i];
	const float u = (float)*p, w = (float)*q;
	*p = (T)fmaf(u, c.x, -(w * c.y));
	*q = (T)fmaf(w, c.x, u * c.y);
}

// 64 keys x 32 dimensions of a group per workgroup: rotated keys straight through, values transposed through LDS into the
// key order of the attention operand; keys past the end are zero values
template <class TR>
__global__ __launch_bounds__(256) void key_values_kernel(TgKeyValues a) {
	typedef typename TR::T T;
	__shared__ T s_v[32][64 + 4];
	const int grp = blockIdx.y, d0 = blockIdx.z * 32, k0 = blockIdx.x * 64, tid = threadIdx.x;
	const int rowp = a.dimp + a.rotp;
	for (int e = tid; e < 64 * 32; e += 256) {
		const int kk = e >> 5, d = e & 31, key = k0 + kk;
		T v = (T)0.0f;
		if (key < a.n) {
			const T *row = (const T *)a.cache + ((size_t)(a.lo + key) * a.groups + grp) * rowp;
			v = row[d0 + d];
			((T *)a.k)[(size_t)key * a.groups * a.dimp + (size_t)grp * a.dimp + d0 + d] = d0 + d < a.rot_size ? row[a.dimp + d0 + d] : v;
		}
		int at = kk;
		if constexpr (TR::DT == TG_DT_BF16) at = (kk & 32) + 8 * ((kk & 15) >> 2) + 4 * ((kk >> 4) & 1) + (kk & 3);
		s_v[d][at] = v;
	}
	__syncthreads();
	for (int e = tid; e < 64 * 32; e += 256) {
		const int d = e >> 6, at = e & 63;
		((T *)a.vt)[(size_t)(grp * a.dimp + d0 + d) * a.ldv + k0 + at] = s_v[d][at];
	}
}

// A workgroup: one head, 64 QT queries (wave: 16 QT of them).  Per tile of KT keys: K and V^T fragments go global ->
// registers -> LDS, the next tile's loads in flight during this one's arithmetic.  Scores are taken as K Q^T, so a lane holds
// four consecutive keys of one query and the probabilities are already the second operand of V^T P^T; in the bf16 format they
// enter it as two bf16 planes (value and remainder).
// Sizes are compile-time buckets (DM >= dimp, VM >= vdimp): query elements past the head are zero, value rows past it are
// computed from repeated rows and not stored, so that no branch stands between the LDS reads and matrix instructions.
// WIDE: with a window, a rotated part or grouped heads.
template <class TR, int DM, int VM, int KT, int QT, bool WIDE>
__global__ __launch_bounds__(256, 2) void latent_attn_kernel(TgLatentRows a) {
	typedef typename TR::T T;
	typedef typename TR::Frag Frag;
	constexpr int ND = DM / TR::KF, NV = VM / 16, NK = KT / 16, NB = KT / TR::KF;
	constexpr int KFRAGS = NK * ND, NF = KFRAGS + NV * NB, PW = NF / 4;
	static_assert(NF % 4 == 0 && NB >= 1, "");
	__shared__ __align__(16) Frag lds[NF * 64];
	const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, lr = lane & 15, lg = lane >> 4;
	// Query tiles from both ends: the first half of the launch takes the long rows, longest first, the second half the
	// short ones, shortest first, so that the workgroups that meet on a compute unit have about the same work together.
	const int nqt = (int)gridDim.y, y = (int)blockIdx.y, half = (nqt + 1) / 2;
	const int h = blockIdx.x, kh = WIDE ? h / a.group : h, qb = (y < half ? nqt - 1 - y : y - half) * 64 * QT;
	const int kn = a.dimp / TR::KF, kd = (a.dimp + (WIDE ? a.rotp : 0)) / TR::KF, nv = a.vdimp / 16;
	const T *Q = (const T *)a.q, *K = (const T *)a.k + (size_t)kh * a.dimp, *V = (const T *)a.vt + (size_t)kh * a.vdimp * a.ldv;
	const T *R = (const T *)a.kr;
	const float sl2 = fabsf(a.scale) * 1.44269504088896340736f;  // (the sign goes to the queries: maxima are taken before scaling)
	const bool neg = a.scale < 0.0f;

	Frag qf[QT][ND];
	int qi[QT];
#pragma unroll
	for (int s = 0; s < QT; s++) {
		qi[s] = qb + w * 16 * QT + s * 16 + lr;
		const T *row = Q + (size_t)min(qi[s], a.n - 1) * a.ldq + (size_t)h * (a.dimp + (WIDE ? a.rotp : 0)) + lg * TR::KV;
#pragma unroll
		for (int d = 0; d < ND; d++) {
			qf[s][d] = *reinterpret_cast<const Frag *>(row + (d < kd ? d : 0) * TR::KF);
			if (d >= kd) qf[s][d] = Frag{};
			if (neg) qf[s][d] = -qf[s][d];
		}
	}
	f32x4_t o[QT][NV];
	float m[QT], l[QT];
#pragma unroll
	for (int s = 0; s < QT; s++) {
		m[s] = -1e30f;  // below every score; finite, so that a tile without a visible key leaves everything as it is
		l[s] = 0.0f;
#pragma unroll
		for (int v = 0; v < NV; v++) o[s][v] = f32x4_t{0, 0, 0, 0};
	}
	const int last = a.past + min(qb + 64 * QT, a.n) - 1;  // the last key any of these queries sees
	const int nt = last / KT + 1, ctx = a.past + a.n, tb = WIDE ? max(a.past + qb - a.window + 1, 0) / KT : 0;
	Frag st[PW];
	auto fetch = [&](int k0) {
#pragma unroll
		for (int i = 0; i < PW; i++) {
			const int f = i * 4 + w;
			const T *p;
			if (f < KFRAGS) {
				const int kt = f / ND, d = f % ND;
				const size_t key = (size_t)min(k0 + kt * 16 + lr, ctx - 1);
				if constexpr (!WIDE) p = K + key * a.ldk + (d < kd ? d : 0) * TR::KF + lg * TR::KV;
				else p = (d < kn || d >= kd ? K + key * a.ldk + (d < kn ? d : 0) * TR::KF : R + key * a.ldkr + (d - kn) * TR::KF) + lg * TR::KV;
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
	fetch(tb * KT);
	put();
	tg_lds_barrier();
	for (int t = tb; t < nt; t++) {
		const int k0 = t * KT;
		fetch((t + 1 < nt ? t + 1 : t) * KT);
		f32x4_t sc[QT][NK];
#pragma unroll
		for (int kt = 0; kt < NK; kt++) {
#pragma unroll
			for (int s = 0; s < QT; s++) sc[s][kt] = f32x4_t{0, 0, 0, 0};
#pragma unroll
			for (int d = 0; d < ND; d++) {
				const Frag kf = lds[(kt * ND + d) * 64 + lane];
#pragma unroll
				for (int s = 0; s < QT; s++) sc[s][kt] = TR::mma(kf, qf[s][d], sc[s][kt]);
			}
		}
		// keys past a query only in the tiles that reach the wave's first query, keys before its window in those that do not
		// reach the last query's
		const int first_q = a.past + qb + w * 16 * QT;
		const bool masked = k0 + KT - 1 > first_q || (WIDE && k0 < first_q + 16 * QT - a.window);
#pragma unroll
		for (int s = 0; s < QT; s++) {
			if (masked) {
				const int lim = a.past + qi[s] - k0 - 4 * lg, low = WIDE ? lim - a.window : -TG_NO_WINDOW;
#pragma unroll
				for (int kt = 0; kt < NK; kt++)
#pragma unroll
					for (int e = 0; e < 4; e++) sc[s][kt][e] = kt * 16 + e <= lim && (!WIDE || kt * 16 + e > low) ? sc[s][kt][e] : -INFINITY;
			}
			float mt = -INFINITY;
#pragma unroll
			for (int kt = 0; kt < NK; kt++)
#pragma unroll
				for (int e = 0; e < 4; e++) mt = fmaxf(mt, sc[s][kt][e]);
			mt = fmaxf(mt, tg_red_partner<32>(mt));
			mt = fmaxf(mt, tg_red_partner<16>(mt));
			const float mn = fmaxf(m[s], mt * sl2);
			if (__ballot(mn > m[s])) {
				const float f = __builtin_amdgcn_exp2f(m[s] - mn);
				l[s] *= f;
#pragma unroll
				for (int v = 0; v < NV; v++)
#pragma unroll
					for (int e = 0; e < 4; e++) o[s][v][e] *= f;
				m[s] = mn;
			}
			float sum = 0.0f;
#pragma unroll
			for (int kt = 0; kt < NK; kt++)
#pragma unroll
				for (int e = 0; e < 4; e++) {
					const float p = __builtin_amdgcn_exp2f(fmaf(sc[s][kt][e], sl2, -mn));
					sc[s][kt][e] = p;
					sum += p;
				}
			l[s] += sum;
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
			for (int v = 0; v < NV; v++) {
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
		const float f = (a.gate ? tg_sigmoid(a.gate[(size_t)qi[s] * a.ld_gate + h]) : 1.0f) / ls;
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

template <class TR, int DM, int VM, int KT, bool WIDE>
void launch_bucket_w(const TgLatentRows &a, hipStream_t s) {
	// 128-query tiles (half the LDS reads per product) where they fill the device twice
	if constexpr (TR::DT == TG_DT_BF16 && DM <= 128 && VM <= 128) {
		if (a.heads * ((a.n + 127) / 128) >= 512) {
			hipLaunchKernelGGL((latent_attn_kernel<TR, DM, VM, KT, 2, WIDE>), dim3((unsigned)a.heads, (unsigned)((a.n + 127) / 128)), dim3(256), 0, s, a);
			return;
		}
	}
	hipLaunchKernelGGL((latent_attn_kernel<TR, DM, VM, KT, 1, WIDE>), dim3((unsigned)a.heads, (unsigned)((a.n + 63) / 64)), dim3(256), 0, s, a);
}
template <class TR, int DM, int VM, int KT>
void launch_bucket(const TgLatentRows &a, hipStream_t s) {
	if (a.rotp || a.group > 1 || a.window < TG_NO_WINDOW) launch_bucket_w<TR, DM, VM, KT, true>(a, s);
	else launch_bucket_w<TR, DM, VM, KT, false>(a, s);
}

template <class TR>
void launch_attention(const TgLatentRows &a, hipStream_t s) {
	constexpr int W = TR::DT == TG_DT_BF16 ? 64 : 32;  // keys per tile of the wide buckets
	const int d = a.dimp + a.rotp, v = a.vdimp;
	if (d <= 64 && v <= 64) launch_bucket<TR, 64, 64, 64>(a, s);
	else if (d <= 64 && v <= 128) launch_bucket<TR, 64, 128, 64>(a, s);
	else if (d <= 128 && v <= 64) launch_bucket<TR, 128, 64, 64>(a, s);
	else if (d <= 128 && v <= 128) launch_bucket<TR, 128, 128, W>(a, s);
	else if (d <= 192 && v <= 128) launch_bucket<TR, 192, 128, 32>(a, s);
	else launch_bucket<TR, 256, 256, 32>(a, s);
}

}  // namespace

namespace {
template <class TR>
void launch_step(const TgLatentStep &a, hipStream_t s) {
	const dim3 grid((unsigned)a.nb, (unsigned)(a.groups * ((a.heads + 15) / 16)), (unsigned)((a.rankp + 511) / 512));
	const size_t lds = latent_step_lds<TR>(a.rowp());
	auto go = [&](auto *kernel) {
		if (lds > 48 * 1024) (void)hipFuncSetAttribute((const void *)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
		hipLaunchKernelGGL(kernel, grid, dim3(256), lds, s, a);
	};
	if (a.rotp && a.rankp <= 128) go(latent_step_kernel<TR, true, 2>);
	else if (a.rotp && a.rankp <= 256) go(latent_step_kernel<TR, true, 4>);
	else if (a.rotp) go(latent_step_kernel<TR, true, 8>);
	else if (a.rankp <= 256) go(latent_step_kernel<TR, false, 4>);
	else go(latent_step_kernel<TR, false, 8>);
}
}  // namespace

void tg_launch_latent_step(const TgLatentStep &a, int dt, hipStream_t s) {
	if (dt == TG_DT_BF16) launch_step<TgB16>(a, s);
	else launch_step<TgF32>(a, s);
}

size_t tg_latent_step_lds(int rowp, int dt) { return dt == TG_DT_BF16 ? latent_step_lds<TgB16>(rowp) : latent_step_lds<TgF32>(rowp); }

void tg_launch_latent_fold(const float *acc, const float *ml, int nb, int heads_padded, int rankp, float *out_acc, float *out_ml, hipStream_t s) {
	hipLaunchKernelGGL(latent_fold_kernel, dim3((unsigned)heads_padded, (unsigned)((rankp + 63) / 64)), dim3(256), 0, s, acc, ml, nb, heads_padded, rankp,
	                   out_acc, out_ml, 0, 1, 0);
}

void tg_launch_latent_finish(const float *acc, const float *ml, int nb, int groups, int heads, int rankp, float *out, int out_stride, hipStream_t s) {
	hipLaunchKernelGGL(latent_fold_kernel, dim3((unsigned)(groups * heads), (unsigned)((rankp + 63) / 64)), dim3(256), 0, s, acc, ml, nb,
	                   groups * tg_up(heads, 16), rankp, out, (float *)nullptr, groups, heads, out_stride);
}

namespace {
template <class TR>
void launch_cache_rows(const TgLatentCacheRows &a, hipStream_t s) {
	const dim3 grid((unsigned)((a.n * a.groups + 3) / 4));
	if (a.f32) hipLaunchKernelGGL((latent_rows_kernel<TR, float>), grid, dim3(256), 0, s, a);
	else hipLaunchKernelGGL((latent_rows_kernel<TR, typename TR::T>), grid, dim3(256), 0, s, a);
}
}  // namespace

void tg_launch_latent_rows(const TgLatentCacheRows &a, int dt, hipStream_t s) {
	if (dt == TG_DT_BF16) launch_cache_rows<TgB16>(a, s);
	else launch_cache_rows<TgF32>(a, s);
}

void tg_launch_rot_rows(void *rows, int ld, int n, int past, int first, int count, int stride, const TgRot &rot, int dt, hipStream_t s) {
	const dim3 grid((unsigned)((count * (rot.dims / 2) + 255) / 256), (unsigned)n);
	if (dt == TG_DT_BF16) hipLaunchKernelGGL((rot_rows_kernel<__bf16>), grid, dim3(256), 0, s, (__bf16 *)rows, ld, past, first, count, stride, rot);
	else hipLaunchKernelGGL((rot_rows_kernel<float>), grid, dim3(256), 0, s, (float *)rows, ld, past, first, count, stride, rot);
}

void tg_launch_key_values(const TgKeyValues &a, int dt, hipStream_t s) {
	const dim3 grid((unsigned)((a.n + 63) / 64), (unsigned)a.groups, (unsigned)(a.dimp / 32));
	if (dt == TG_DT_BF16) hipLaunchKernelGGL((key_values_kernel<TgB16>), grid, dim3(256), 0, s, a);
	else hipLaunchKernelGGL((key_values_kernel<TgF32>), grid, dim3(256), 0, s, a);
}

void tg_launch_latent_attention(const TgLatentRows &a, int dt, hipStream_t s) {
	if (dt == TG_DT_BF16) launch_attention<TgB16>(a, s);
	else launch_attention<TgF32>(a, s);
}
