// Gated linear attention and the gated delta rule: the step of one token, and the chunked form of many (tg_gla.h).
//
// Chunked form.  With b_t the sum of log alpha over the chunk's tokens up to and including t, a chunk of 64 tokens that
// starts from state S contributes
//     o_i = (q_i e^{b_i})^T S + sum_{j <= i} A_ij v_j,   A_ij = sum_d q_id k_jd e^{b_id - b_jd},
//     S'  = diag(e^{b_end}) S + sum_j (k_j e^{b_end - b_j}) v_j^T
// (b is kept in units of log 2, so every exponential is one v_exp_f32), all exponents <= 0, whatever the decay: A's blocks of 16 x 16 below the diagonal take the exponent apart at the row
// block's first token (both halves <= 0) and run on the fp32 matrix instructions, the diagonal blocks are summed pair by
// pair.  Four launches: b; A and the chunks' own state contributions U, all chunks at once; the states in front of every
// chunk, one pass over U; the outputs, all chunks at once.  Everything is fp32 (q, k, v are read in the model's format).

#include "tg_gla.h"

namespace {

constexpr int C = TG_GLA_CHUNK;
__device__ __forceinline__ float pow2(float x) { return __builtin_amdgcn_exp2f(x); }

// ---- one token -----------------------------------------------------------------------------------------------------------
// A workgroup owns 32 value columns of a head: lane = 4 columns, 32 groups of key channels.
__global__ __launch_bounds__(256) void gla_step_kernel(const float *y, TgGla g, int k_off, int v_off, int a_off, float *o) {
	extern __shared__ __align__(16) float sm[];
	float *s_q = sm, *s_k = sm + g.dimp, *s_a = sm + 2 * g.dimp;
	__shared__ f32x4_t s_red[4][8];
	const int h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
	const int col = blockIdx.y * 32 + (tid & 7) * 4, dg = tid >> 3, hd = g.heads * g.dimp;
	float *S = g.state + ((size_t)h * g.dimp) * g.vdimp + col;
	f32x4_t st[4];
	const f32x4_t v = tg_load4(y + v_off + (size_t)h * g.vdimp + col);
#pragma unroll
	for (int r = 0; r < 4; r++) st[r] = tg_load4(S + (size_t)min(dg + 32 * r, g.dimp - 1) * g.vdimp);
	for (int d = tid; d < g.dimp; d += 256) {
		const size_t c = (size_t)h * g.dimp + d;
		float z = 0.0f;
		for (int j0 = 0; j0 < g.rank; j0 += 16) {
			float wa[16], ya[16];
#pragma unroll
			for (int j = 0; j < 16; j++) {
				wa[j] = g.a2[(size_t)min(j0 + j, g.rank - 1) * hd + c];
				ya[j] = y[a_off + min(j0 + j, g.rank - 1)];
			}
#pragma unroll
			for (int j = 0; j < 16; j++) z = j0 + j < g.rank ? fmaf(wa[j], ya[j], z) : z;
		}
		s_a[d] = pow2(tg_log2_sigmoid(z + g.a2b[c]) * g.inv_tau);
		s_q[d] = y[c] * g.qscale;
		s_k[d] = y[k_off + c];
	}
	__syncthreads();
	f32x4_t acc = {0, 0, 0, 0};
	for (int d0 = 0; d0 < g.dimp; d0 += 128) {
#pragma unroll
		for (int r = 0; r < 4; r++) {
			const int d = d0 + dg + 32 * r;
			if (d0) st[r] = tg_load4(S + (size_t)min(d, g.dimp - 1) * g.vdimp);
			if (d < g.dimp) {
				const float a = s_a[d], k = s_k[d], q = s_q[d];
#pragma unroll
				for (int e = 0; e < 4; e++) {
					st[r][e] = fmaf(a, st[r][e], k * v[e]);
					acc[e] = fmaf(q, st[r][e], acc[e]);
				}
				tg_store4(S + (size_t)d * g.vdimp, st[r]);
			}
		}
	}
#pragma unroll
	for (int e = 0; e < 4; e++) {
		acc[e] += tg_red_partner<32>(acc[e]);
		acc[e] += tg_red_partner<16>(acc[e]);
		acc[e] += tg_red_partner<8>(acc[e]);
	}
	if (lane < 8) s_red[w][lane] = acc;
	__syncthreads();
	if (tid < 8) {
		f32x4_t r = s_red[0][tid];
#pragma unroll
		for (int i = 1; i < 4; i++)
#pragma unroll
			for (int e = 0; e < 4; e++) r[e] += s_red[i][tid][e];
		tg_store4(o + (size_t)h * g.vdimp + col, r);
	}
}

// ---- running sums of log alpha inside every chunk: 64 channels per workgroup, a wave per 16 tokens ----------------------------
__global__ __launch_bounds__(256) void gla_decay_kernel(const float *low, int ld_low, TgGla g, int n, float *b) {
	__shared__ __align__(16) float s_low[C][20];
	__shared__ float s_sum[4][64];
	const int hd = g.heads * g.dimp, tid = threadIdx.x, lane = tid & 63, w = tid >> 6, t0 = blockIdx.x * C;
	const int c = blockIdx.y * 64 + lane, cc = min(c, hd - 1);
	const bool real = c < hd && cc % g.dimp < g.dim;
	// softplus(z) = -log(sigmoid(-z))
	const float bias = g.a2b[cc], flip = g.a_log ? -1.0f : 1.0f, rate = g.a_log ? expf(g.a_log[cc / g.dimp]) : g.inv_tau;
	float z[16];
#pragma unroll
	for (int i = 0; i < 16; i++) z[i] = bias;
	for (int j0 = 0; j0 < g.rank; j0 += 16) {
		float wj[16];
#pragma unroll
		for (int j = 0; j < 16; j++) wj[j] = g.a2[(size_t)min(j0 + j, g.rank - 1) * hd + cc];
		// (the rows of `low` are padded to a multiple of 16)
		const f32x4_t v = tg_load4(low + (size_t)min(t0 + (tid >> 2), n - 1) * ld_low + j0 + (tid & 3) * 4);
		__syncthreads();
		tg_store4(&s_low[tid >> 2][(tid & 3) * 4], v);
		__syncthreads();
#pragma unroll
		for (int j = 0; j < 16; j++)
			if (j0 + j >= g.rank) wj[j] = 0.0f;
#pragma unroll
		for (int i = 0; i < 16; i++)
#pragma unroll
			for (int j4 = 0; j4 < 4; j4++) {
				const f32x4_t l = tg_load4(&s_low[16 * w + i][4 * j4]);
#pragma unroll
				for (int e = 0; e < 4; e++) z[i] = fmaf(wj[4 * j4 + e], l[e], z[i]);
			}
	}
	float run = 0.0f;
#pragma unroll
	for (int i = 0; i < 16; i++) {
		if (real && t0 + 16 * w + i < n) run += tg_log2_sigmoid(flip * z[i]) * rate;  // past the end: the sum stays
		z[i] = run;
	}
	s_sum[w][lane] = run;
	__syncthreads();
	float before = 0.0f;
	for (int q = 0; q < w; q++) before += s_sum[q][lane];
	if (c < hd)
#pragma unroll
		for (int i = 0; i < 16; i++) b[(size_t)(t0 + 16 * w + i) * hd + c] = before + z[i];
}

// ---- A: a workgroup per chunk and head, a wave per block of 16 rows ---------------------------------------------------------
constexpr int SL = 32, SLP = 36;  // key channels per slab, row pitch

// DELTA: also k . k with the decay between them, T = beta (k . k) below the diagonal, of which it leaves -T outside the 16 x 16
// diagonal blocks and in those the inverse of 1 + T's block (by substitution, a lane per column).
struct DeltaIntra {
	const float *beta;  // [n][ld_beta], before the sigmoid
	int ld_beta;
	float *t;           // [chunks][heads][64][64]
};

template <class TR, bool DELTA>
__global__ __launch_bounds__(256) void gla_intra_kernel(const typename TR::T *qkv, int ld, int k_off, TgGla g, int n, const float *b, float *A,
                                                        DeltaIntra x) {
	__shared__ __align__(16) float s_q[C][SLP], s_k[C][SLP], s_b[C][SLP];
	const int ch = blockIdx.x, h = blockIdx.y, kh = DELTA ? h / g.group : h, tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
	const int lr = lane & 15, lg = lane >> 4, hd = g.heads * g.dimp, t0 = ch * C;
	f32x4_t off[3], dia = {0, 0, 0, 0}, koff[3], kdia = {0, 0, 0, 0};
#pragma unroll
	for (int j = 0; j < 3; j++) off[j] = koff[j] = f32x4_t{0, 0, 0, 0};
	for (int d0 = 0; d0 < g.dimp; d0 += SL) {
		__syncthreads();
		for (int e = tid; e < C * SL / 4; e += 256) {
			const int r = e / (SL / 4), c4 = (e % (SL / 4)) * 4, t = t0 + r;
			const size_t col = (size_t)h * g.dimp + d0 + c4, kcol = (size_t)kh * g.dimp + d0 + c4;
			f32x4_t q = tg_load4(qkv + (size_t)min(t, n - 1) * ld + kcol), k = tg_load4(qkv + (size_t)min(t, n - 1) * ld + k_off + kcol);
#pragma unroll
			for (int i = 0; i < 4; i++) {
				q[i] = t < n ? q[i] * g.qscale : 0.0f;
				k[i] = t < n ? k[i] : 0.0f;
			}
			tg_store4(&s_q[r][c4], q);
			tg_store4(&s_k[r][c4], k);
			tg_store4(&s_b[r][c4], tg_load4(b + (size_t)t * hd + col));
		}
		__syncthreads();
		const int qi = 16 * w + lr;
		if (w > 0) {
			for (int st = 0; st < SL / 4; st++) {
				const int d = 4 * st + lg;
				const float ref = s_b[16 * w - 1][d];
				const float fade = pow2(s_b[qi][d] - ref), qv = s_q[qi][d] * fade, kq = DELTA ? s_k[qi][d] * fade : 0.0f;
#pragma unroll
				for (int j = 0; j < 3; j++)
					if (j < w) {
						const float kv = s_k[16 * j + lr][d] * pow2(ref - s_b[16 * j + lr][d]);
						off[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(qv, kv, off[j], 0, 0, 0);
						if constexpr (DELTA) koff[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(kq, kv, koff[j], 0, 0, 0);
					}
			}
		}
		for (int d = 0; d < SL; d += 4) {
			const f32x4_t q = tg_load4(&s_q[qi][d]), bi = tg_load4(&s_b[qi][d]);
			f32x4_t ki = {0, 0, 0, 0};
			if constexpr (DELTA) ki = tg_load4(&s_k[qi][d]);
#pragma unroll
			for (int j = 0; j < 4; j++) {
				const int kj = 16 * w + 4 * lg + j;
				const f32x4_t k = tg_load4(&s_k[kj][d]), bj = tg_load4(&s_b[kj][d]);
				if (kj <= qi) {
#pragma unroll
					for (int e = 0; e < 4; e++) {
						const float fade = pow2(bi[e] - bj[e]);
						dia[j] = fmaf(q[e] * k[e], fade, dia[j]);
						if constexpr (DELTA) kdia[j] = fmaf(ki[e] * k[e], fade, kdia[j]);
					}
				}
			}
		}
	}
	float *out = A + ((size_t)ch * g.heads + h) * C * C;
#pragma unroll
	for (int j = 0; j < 4; j++) {
		if (j == w) {
			tg_store4(out + (size_t)(16 * w + lr) * C + 16 * w + 4 * lg, dia);
		} else {
#pragma unroll
			for (int e = 0; e < 4; e++) out[(size_t)(16 * w + 4 * lg + e) * C + 16 * j + lr] = j < w ? off[j < 3 ? j : 0][e] : 0.0f;
		}
	}
	if constexpr (DELTA) {
		__shared__ __align__(16) float s_t[4][16][20];
		float *T = x.t + ((size_t)ch * g.heads + h) * C * C;
		float beta_q = 0.0f, beta_r[4];
		auto step = [&](int r) { return t0 + r < n ? tg_sigmoid(x.beta[(size_t)(t0 + r) * x.ld_beta + h]) : 0.0f; };
		beta_q = step(16 * w + lr);
#pragma unroll
		for (int e = 0; e < 4; e++) beta_r[e] = step(16 * w + 4 * lg + e);
#pragma unroll
		for (int j = 0; j < 4; j++) s_t[w][lr][4 * lg + j] = 4 * lg + j < lr ? beta_q * kdia[j] : 0.0f;
#pragma unroll
		for (int j = 0; j < 3; j++)
			if (j < w) {
#pragma unroll
				for (int e = 0; e < 4; e++) T[(size_t)(16 * w + 4 * lg + e) * C + 16 * j + lr] = -beta_r[e] * koff[j][e];
			}
		__syncthreads();
		float m[16];
#pragma unroll
		for (int r = 0; r < 16; r++) {
			float v = r == lr ? 1.0f : 0.0f;
			f32x4_t tr[4];
#pragma unroll
			for (int j = 0; j < 4; j++) tr[j] = tg_load4(&s_t[w][r][4 * j]);
#pragma unroll
			for (int j = 0; j < r; j++) v = fmaf(-tr[j >> 2][j & 3], m[j], v);
			m[r] = v;
		}
		if (lg == 0)
#pragma unroll
			for (int r = 0; r < 16; r++) T[(size_t)(16 * w + r) * C + 16 * w + lr] = m[r];
	}
}

// ---- the chunk's solved keys and values (delta rule): u = M (beta v) - M (beta k e^b) S with M = (1 + T)^-1, S the state in front of it -
// The solve runs down the 16 x 16 blocks on the matrix instructions, a wave per two tiles of 16 columns: an accumulator (four
// consecutive rows of a column per lane) is the next product's second operand as it is, with the first operand's columns taken
// in the same order.  Also the keys decayed to the chunk's end, transposed.
// Results lie in operand order, 16 x 16 tiles of [lane][4]: wk in tiles (key channels, tokens), lane = token % 16 + 16 (channel % 16
// / 4), the four values being consecutive channels (turned through LDS); kt and u in tiles (key channels or value columns, tokens),
// lane = channel % 16 + 16 (token % 16 / 4), consecutive tokens.
struct DeltaSolve {
	const float *qk, *b, *t, *beta;
	int ldqk, k_off, ld_beta;
	const float *v;
	float *u, *wk, *kt;
};
__global__ __launch_bounds__(256) void delta_solve_kernel(DeltaSolve x, TgGla g, int n) {
	__shared__ __align__(16) float s_beta[C], s_turn[4][16][20];
	const int ch = blockIdx.x, h = blockIdx.y, kh = h / g.group, tid = threadIdx.x, lane = tid & 63, w = tid >> 6, lr = lane & 15, lg = lane >> 4;
	const int hd = g.heads * g.dimp, hv = g.heads * g.vdimp, t0 = ch * C;
	const int nk = g.dimp / 16, ntile = nk + g.vdimp / 16, tile0 = ((int)blockIdx.z * 4 + w) * 2;
	const float *T = x.t + ((size_t)ch * g.heads + h) * C * C;
	const float raw = x.beta[(size_t)min(t0 + (tid & 63), n - 1) * x.ld_beta + h];
	f32x4_t tb[6], mb[4];  // blocks (1,0) (2,0) (2,1) (3,0) (3,1) (3,2); the inverses
#pragma unroll
	for (int i = 0; i < 4; i++) {
		mb[i] = tg_load4(T + (size_t)(16 * i + lr) * C + 16 * i + 4 * lg);
#pragma unroll
		for (int j = 0; j < i; j++) tb[i * (i - 1) / 2 + j] = tg_load4(T + (size_t)(16 * i + lr) * C + 16 * j + 4 * lg);
	}
	// (a wave past the last tile repeats it and stores nothing; tiles come in pairs: nk and the number of value tiles are even)
	const bool live = tile0 < ntile;
	const int tile = live ? tile0 : ntile - 2;
	const bool key = tile < nk;
	int col[2];
	f32x4_t X[2][4], W[2][4], bt[2][4];
	float be[2] = {0.0f, 0.0f};
#pragma unroll
	for (int p = 0; p < 2; p++) {
		col[p] = (key ? tile : tile - nk) * 16 + 16 * p + lr;
		const float *src = key ? x.qk + x.k_off + (size_t)kh * g.dimp + col[p] : x.v + (size_t)h * g.vdimp + col[p];
		const int ld = key ? x.ldqk : hv;
#pragma unroll
		for (int i = 0; i < 4; i++)
#pragma unroll
			for (int e = 0; e < 4; e++) X[p][i][e] = src[(size_t)min(t0 + 16 * i + 4 * lg + e, n - 1) * ld];
		if (key) {
			const float *bp = x.b + (size_t)t0 * hd + (size_t)h * g.dimp + col[p];
			be[p] = bp[(size_t)(C - 1) * hd];
#pragma unroll
			for (int i = 0; i < 4; i++)
#pragma unroll
				for (int e = 0; e < 4; e++) bt[p][i][e] = bp[(size_t)(16 * i + 4 * lg + e) * hd];
		}
	}
	if (tid < C) s_beta[tid] = t0 + tid < n ? tg_sigmoid(raw) : 0.0f;
	__syncthreads();
#pragma unroll
	for (int p = 0; p < 2; p++)
#pragma unroll
		for (int i = 0; i < 4; i++) {
			const f32x4_t beta = tg_load4(&s_beta[16 * i + 4 * lg]);
			if (key) {
				f32x4_t kd;
#pragma unroll
				for (int e = 0; e < 4; e++) {
					kd[e] = t0 + 16 * i + 4 * lg + e < n ? X[p][i][e] * pow2(be[p] - bt[p][i][e]) : 0.0f;
					X[p][i][e] *= pow2(bt[p][i][e]);
				}
				if (live) tg_store4(x.kt + (size_t)t0 * hd + (size_t)h * g.dimp * C + (((tile + p) * 4 + i) * 64 + lane) * 4, kd);
			}
#pragma unroll
			for (int e = 0; e < 4; e++) X[p][i][e] *= beta[e];
		}
#pragma unroll
	for (int i = 0; i < 4; i++) {
#pragma unroll
		for (int j = 0; j < i; j++)
#pragma unroll
			for (int e = 0; e < 4; e++)
#pragma unroll
				for (int p = 0; p < 2; p++) X[p][i] = __builtin_amdgcn_mfma_f32_16x16x4f32(tb[i * (i - 1) / 2 + j][e], W[p][j][e], X[p][i], 0, 0, 0);
#pragma unroll
		for (int p = 0; p < 2; p++) W[p][i] = f32x4_t{0, 0, 0, 0};
#pragma unroll
		for (int e = 0; e < 4; e++)
#pragma unroll
			for (int p = 0; p < 2; p++) W[p][i] = __builtin_amdgcn_mfma_f32_16x16x4f32(mb[i][e], X[p][i][e], W[p][i], 0, 0, 0);
	}
	if (!live) return;
#pragma unroll
	for (int p = 0; p < 2; p++) {
		float *dst = key ? x.wk + (size_t)t0 * hd + (size_t)h * g.dimp * C + (tile + p) * 1024 : x.u + (size_t)t0 * hv + (size_t)h * g.vdimp * C + (tile - nk + p) * 1024;
#pragma unroll
		for (int i = 0; i < 4; i++) {
			if (key) {
#pragma unroll
				for (int e = 0; e < 4; e++) s_turn[w][4 * lg + e][lr] = W[p][i][e];
				__builtin_amdgcn_wave_barrier();
				W[p][i] = tg_load4(&s_turn[w][lr][4 * lg]);
				__builtin_amdgcn_wave_barrier();
			}
			tg_store4(dst + (i * 64 + lane) * 4, W[p][i]);
		}
	}
}

// ---- U = sum_j (k_j e^{b_end - b_j}) v_j^T: 128 key channels x VB value columns per workgroup, 8 waves of 64 x VB / 4 -----------
template <class TR, int VB>
__global__ __launch_bounds__(512) void gla_state_kernel(const typename TR::T *qkv, int ld, int k_off, int v_off, TgGla g, int n, const float *b,
                                                        float *U) {
	constexpr int KP = 128 + 16, VP = VB + 16, NI = VB / 64;  // pitches: four rows side by side meet all banks
	__shared__ __align__(16) float s_k[C][KP], s_v[C][VP];
	const int ch = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, w = tid >> 6, wd = (w & 1) * 64, wv = (w >> 1) * (VB / 4);
	const int nvb = (g.vdimp + VB - 1) / VB, d0 = (int)(blockIdx.z / nvb) * 128, v0 = (int)(blockIdx.z % nvb) * VB;
	const int lr = lane & 15, lg = lane >> 4, hd = g.heads * g.dimp, t0 = ch * C;
#pragma unroll
	for (int i = 0; i < C * 32 / 512; i++) {
		const int e = tid + 512 * i, r = e >> 5, c4 = (e & 31) * 4, t = t0 + r, tc = min(t, n - 1);
		const bool in = t < n && d0 + c4 < g.dimp;
		const size_t kc = (size_t)h * g.dimp + (in ? d0 + c4 : 0);
		const f32x4_t k = tg_load4(qkv + (size_t)tc * ld + k_off + kc);
		const f32x4_t be = tg_load4(b + (size_t)(t0 + C - 1) * hd + kc), bj = tg_load4(b + (size_t)t * hd + kc);
		f32x4_t ks;
#pragma unroll
		for (int q = 0; q < 4; q++) ks[q] = in ? k[q] * pow2(be[q] - bj[q]) : 0.0f;
		tg_store4(&s_k[r][c4], ks);
	}
#pragma unroll
	for (int i = 0; i < C * VB / 4 / 512; i++) {
		const int e = tid + 512 * i, r = e / (VB / 4), c4 = (e % (VB / 4)) * 4, t = t0 + r, tc = min(t, n - 1);
		const bool in = t < n && v0 + c4 < g.vdimp;
		f32x4_t v = tg_load4(qkv + (size_t)tc * ld + v_off + (size_t)h * g.vdimp + (in ? v0 + c4 : 0));
		if (!in) v = f32x4_t{0, 0, 0, 0};
		tg_store4(&s_v[r][c4], v);
	}
	__syncthreads();
	f32x4_t acc[4][NI];
#pragma unroll
	for (int i = 0; i < 4; i++)
#pragma unroll
		for (int j = 0; j < NI; j++) acc[i][j] = f32x4_t{0, 0, 0, 0};
#pragma unroll 4
	for (int t = 0; t < C; t += 4) {
		float a[4], v[NI];
#pragma unroll
		for (int i = 0; i < 4; i++) a[i] = s_k[t + lg][wd + 16 * i + lr];
#pragma unroll
		for (int j = 0; j < NI; j++) v[j] = s_v[t + lg][wv + 16 * j + lr];
		// value columns are the first operand: a lane holds four of them for one key channel
#pragma unroll
		for (int i = 0; i < 4; i++)
#pragma unroll
			for (int j = 0; j < NI; j++) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(v[j], a[i], acc[i][j], 0, 0, 0);
	}
	float *out = U + ((size_t)ch * g.heads + h) * g.dimp * g.vdimp;
#pragma unroll
	for (int i = 0; i < 4; i++)
#pragma unroll
		for (int j = 0; j < NI; j++) {
			const int d = d0 + wd + 16 * i + lr, v = v0 + wv + 16 * j + 4 * lg;
			if (d < g.dimp && v < g.vdimp) tg_store4(out + (size_t)d * g.vdimp + v, acc[i][j]);
		}
}

// ---- U becomes the state in front of its chunk; the state behind the last chunk goes to the sequence ---------------------------
__global__ __launch_bounds__(256) void gla_scan_kernel(float *U, const float *b, TgGla g, int chunks) {
	constexpr int AHEAD = 8;  // chunks whose loads are in flight
	const size_t per = (size_t)g.heads * g.dimp * g.vdimp, e = (size_t)blockIdx.x * 256 + threadIdx.x;
	if (e >= per) return;
	const int hd = g.heads * g.dimp, c = (int)(e / g.vdimp);
	float s = g.state[e], u[AHEAD], bn[AHEAD];
	auto load = [&](int i, int ch) {
		ch = min(ch, chunks - 1);
		u[i] = U[(size_t)ch * per + e];
		bn[i] = b[(size_t)(ch * C + C - 1) * hd + c];
	};
#pragma unroll
	for (int i = 0; i < AHEAD; i++) load(i, i);
	for (int ch = 0; ch < chunks; ch += AHEAD) {
#pragma unroll
		for (int i = 0; i < AHEAD; i++) {
			if (ch + i < chunks) {
				U[(size_t)(ch + i) * per + e] = s;
				s = fmaf(pow2(bn[i]), s, u[i]);
			}
			load(i, ch + i + AHEAD);  // (past the end: the last chunk again, unused)
		}
	}
	g.state[e] = s;
}

// ---- o = (q e^b)^T S + A v, the head's root mean square norm and silu(gate): 64 tokens x the whole head per workgroup -------------
// 8 waves: 16 tokens x half of the value columns each.  Slabs of 32: first the key channels (rows q e^b, columns of S), then
// the chunk's own tokens (rows A, columns v); a slab's loads are in flight during the one before it.
// (delta rule: v is u, the states are tiles (value columns, key channels) like u's, the gate's function is the sigmoid)
struct OutIn {
	const void *q, *v, *gate;
	int ldq, ldv, ldg;
};
template <class TI, class TR, int VB, bool DELTA>
__global__ __launch_bounds__(512) void gla_out_kernel(OutIn in, TgGla g, int n, const float *b, const float *A, const float *U, typename TR::T *out,
                                                      int ld_out) {
	const typename TI::T *Q = (const typename TI::T *)in.q + (size_t)(DELTA ? blockIdx.y / g.group : blockIdx.y) * g.dimp,
	                     *V = (const typename TI::T *)in.v + (DELTA ? ((size_t)blockIdx.x * g.heads + blockIdx.y) * g.vdimp * C : (size_t)blockIdx.y * g.vdimp);
	// (delta rule: v and S come transposed and are turned on their way into LDS; the pitch keeps those writes apart)
	constexpr int XP = 36, YP = VB + (DELTA ? 18 : 16), NI = VB / 32, NY = 32 * VB / 4 / 512;
	__shared__ __align__(16) float s_x[C][XP], s_y[32][YP];
	__shared__ float s_sq[2][C];
	const int ch = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, w = tid >> 6, wt = (w & 3) * 16, wv = (w >> 2) * (VB / 2);
	const int lr = lane & 15, lg = lane >> 4, hd = g.heads * g.dimp, t0 = ch * C;
	const float *S = U + ((size_t)ch * g.heads + h) * g.dimp * g.vdimp;
	const int slabs = g.dimp / 32;  // dimp is a multiple of 32
	f32x4_t x, bx, y[NY];
	const int xr = tid >> 3, xc = (tid & 7) * 4;
	auto fetch = [&](int sl) {
		if (sl < slabs) {
			const size_t qc = (size_t)h * g.dimp + sl * 32 + xc;
			x = tg_load4(Q + (size_t)min(t0 + xr, n - 1) * in.ldq + sl * 32 + xc);
			bx = tg_load4(b + (size_t)(t0 + xr) * hd + qc);
#pragma unroll
			for (int i = 0; i < NY; i++) {
				const int e = tid + 512 * i, r = e / (VB / 4), c4 = (e % (VB / 4)) * 4;
				if constexpr (DELTA) y[i] = tg_load4(S + ((size_t)(min(e >> 3, g.vdimp - 1) >> 4) * (g.dimp / 16) + sl * 2 + ((e >> 2) & 1)) * 256 + ((e >> 3) & 15) * 4 + (e & 3) * 64);
				else y[i] = tg_load4(S + (size_t)(sl * 32 + r) * g.vdimp + (c4 < g.vdimp ? c4 : 0));
			}
		} else {
			const int j0 = (sl - slabs) * 32;
			x = tg_load4(A + (((size_t)ch * g.heads + h) * C + xr) * C + j0 + xc);
#pragma unroll
			for (int i = 0; i < NY; i++) {
				const int e = tid + 512 * i, r = e / (VB / 4), c4 = (e % (VB / 4)) * 4;
				if constexpr (DELTA) y[i] = tg_load4(V + ((size_t)(min(e >> 3, g.vdimp - 1) >> 4) * 4 + j0 / 16 + ((e >> 2) & 1)) * 256 + ((e >> 3) & 15) * 4 + (e & 3) * 64);
				else y[i] = tg_load4(V + (size_t)min(t0 + j0 + r, n - 1) * in.ldv + (c4 < g.vdimp ? c4 : 0));
			}
		}
	};
	auto put = [&](int sl) {
		if (sl < slabs) {
#pragma unroll
			for (int e = 0; e < 4; e++) x[e] = x[e] * g.qscale * pow2(bx[e]);
		}
		tg_store4(&s_x[xr][xc], x);
#pragma unroll
		for (int i = 0; i < NY; i++) {
			const int e = tid + 512 * i, r = e / (VB / 4), c4 = (e % (VB / 4)) * 4;
			// (rows of v past the end meet zeros of A)
			if constexpr (DELTA) {
#pragma unroll
				for (int q = 0; q < 4; q++) s_y[(e & 7) * 4 + q][e >> 3] = (e >> 3) < g.vdimp ? y[i][q] : 0.0f;
			} else {
				tg_store4(&s_y[r][c4], c4 < g.vdimp ? y[i] : f32x4_t{0, 0, 0, 0});
			}
		}
	};
	f32x4_t acc[NI];
#pragma unroll
	for (int j = 0; j < NI; j++) acc[j] = f32x4_t{0, 0, 0, 0};
	fetch(0);
	for (int sl = 0; sl < slabs + 2; sl++) {
		put(sl);
		tg_lds_barrier();
		if (sl + 1 < slabs + 2) fetch(sl + 1);
#pragma unroll
		for (int d = 0; d < 32; d += 4) {
			const float a = s_x[wt + lr][d + lg];
#pragma unroll
			for (int j = 0; j < NI; j++) acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(s_y[d + lg][wv + 16 * j + lr], a, acc[j], 0, 0, 0);
		}
		tg_lds_barrier();
	}
	// a lane holds token wt + lr, value columns wv + 16 j + 4 lg ...
	float ss = 0.0f;
#pragma unroll
	for (int j = 0; j < NI; j++)
#pragma unroll
		for (int e = 0; e < 4; e++) ss = fmaf(acc[j][e], acc[j][e], ss);
	ss += tg_red_partner<32>(ss);
	ss += tg_red_partner<16>(ss);
	if (lg == 0) s_sq[w >> 2][wt + lr] = ss;
	__syncthreads();
	const int t = t0 + wt + lr;
	if (t >= n) return;
	const float inv = 1.0f / sqrtf((s_sq[0][wt + lr] + s_sq[1][wt + lr]) / (float)g.vdim + g.eps);
	typename TR::T *dst = out + (size_t)t * ld_out + (size_t)h * g.vdimp;
	const typename TR::T *gate = (const typename TR::T *)in.gate + (size_t)t * in.ldg + (size_t)h * g.vdimp;
#pragma unroll
	for (int j = 0; j < NI; j++) {
		const int v = wv + 16 * j + 4 * lg;
		if (v < g.vdimp) {
			const f32x4_t gv = tg_load4(gate + v), nw = tg_load4(g.norm + v);
			f32x4_t r;
#pragma unroll
			for (int e = 0; e < 4; e++) r[e] = acc[j][e] * inv * nw[e] * (DELTA ? tg_sigmoid(gv[e]) : tg_silu(gv[e]));
			tg_store4(dst + v, r);
		}
	}
	if (h == g.heads - 1)  // the columns behind the heads
		for (int v = g.heads * g.vdimp + (w >> 2) * 16 + 4 * lg; v < ld_out; v += 32) tg_store4(out + (size_t)t * ld_out + v, f32x4_t{0, 0, 0, 0});
}

template <class TI, class TR, int VB, bool DELTA>
void launch_out_vb(const TgGla &g, const OutIn &in, int n, const float *b, const float *A, const float *U, void *out, int ld_out, hipStream_t s) {
	hipLaunchKernelGGL((gla_out_kernel<TI, TR, VB, DELTA>), dim3((unsigned)((n + C - 1) / C), (unsigned)g.heads), dim3(512), 0, s, in, g, n, b, A, U,
	                   (typename TR::T *)out, ld_out);
}
template <class TI, class TR, bool DELTA>
void launch_out(const TgGla &g, const OutIn &in, int n, const float *b, const float *A, const float *U, void *out, int ld_out, hipStream_t s) {
	if (g.vdimp <= 64) launch_out_vb<TI, TR, 64, DELTA>(g, in, n, b, A, U, out, ld_out, s);
	else if (g.vdimp <= 128) launch_out_vb<TI, TR, 128, DELTA>(g, in, n, b, A, U, out, ld_out, s);
	else if (g.vdimp <= 256) launch_out_vb<TI, TR, 256, DELTA>(g, in, n, b, A, U, out, ld_out, s);
	else launch_out_vb<TI, TR, TG_GLA_VDIM_MAX, DELTA>(g, in, n, b, A, U, out, ld_out, s);
}

template <class TR>
void launch_rows(const TgGla &g, const void *qkv, int ld, int k_off, int v_off, int g_off, const float *low, int ld_low, int n,
                 const TgGlaScratch &t, void *out, int ld_out, hipStream_t s) {
	typedef typename TR::T T;
	const T *x = (const T *)qkv;
	const unsigned chunks = (unsigned)((n + C - 1) / C), H = (unsigned)g.heads, hd = (unsigned)(g.heads * g.dimp), nd = (unsigned)((g.dimp + 127) / 128);
	hipLaunchKernelGGL(gla_decay_kernel, dim3(chunks, (hd + 63) / 64), dim3(256), 0, s, low, ld_low, g, n, t.b);
	hipLaunchKernelGGL((gla_intra_kernel<TR, false>), dim3(chunks, H), dim3(256), 0, s, x, ld, k_off, g, n, t.b, t.a, DeltaIntra{});
	if (g.vdimp <= 64)
		hipLaunchKernelGGL((gla_state_kernel<TR, 64>), dim3(chunks, H, nd), dim3(512), 0, s, x, ld, k_off, v_off, g, n, t.b, t.u);
	else
		hipLaunchKernelGGL((gla_state_kernel<TR, 128>), dim3(chunks, H, nd * (unsigned)((g.vdimp + 127) / 128)), dim3(512), 0, s, x, ld, k_off, v_off, g,
		                   n, t.b, t.u);
	const size_t per = (size_t)hd * g.vdimp;
	hipLaunchKernelGGL(gla_scan_kernel, dim3((unsigned)((per + 255) / 256)), dim3(256), 0, s, t.u, t.b, g, (int)chunks);
	launch_out<TR, TR, false>(g, OutIn{x, x + v_off, x + g_off, ld, ld, ld}, n, t.b, t.a, t.u, out, ld_out, s);
}

// ==== the gated delta rule ====================================================================================================
// Chunked form: with the notation above and T_ij = beta_i sum_d k_id k_jd e^{b_id - b_jd} (j < i),
//     (1 + T) u = beta (v - (k e^b)^T S),   o_i = (q_i e^{b_i})^T S + sum_{j <= i} A_ij u_j,
//     S' = diag(e^{b_end}) S + sum_j (k_j e^{b_end - b_j}) u_j^T.
// Launches: convolution and unit norms; b; A, T and the solved keys and values, all chunks at once; the pass over the chunks
// (u and the state in front of each), 16 value columns per workgroup; the outputs, all chunks at once.

// ---- convolution, silu, unit norm: 8 tokens per wave; y: q heads, k heads, blocks of 256 value channels ------------------------------
// Inputs before the portion come from the ring.
// TAPS: the number of taps where it is one of the usual ones (every input row is then read once), else 0.
constexpr int PT = 8;
template <class TR, int TAPS>
__global__ __launch_bounds__(256) void delta_prep_kernel(TgDelta d, const typename TR::T *x, int ld, int n, int past, float *qk, float *v_out) {
	const int t0 = (blockIdx.x * 4 + (threadIdx.x >> 6)) * PT, lane = threadIdx.x & 63, kvh = d.g.heads / d.g.group, qc = d.q_channels();
	if (t0 >= n) return;
	const bool head = (int)blockIdx.y < 2 * kvh;
	const int base = head ? (int)blockIdx.y * d.g.dimp : 2 * qc + ((int)blockIdx.y - 2 * kvh) * 256;
	const int len = head ? d.g.dimp : min(256, d.channels - base);  // (at most 256)
	const int c = base + min(4 * lane, len - 4);
	const bool in = 4 * lane < len;
	f32x4_t r[PT];
#pragma unroll
	for (int p = 0; p < PT; p++) r[p] = f32x4_t{0, 0, 0, 0};
	const bool inside = TAPS > 0 && t0 >= TAPS - 1 && t0 + PT <= n;
	if constexpr (TAPS > 0) {
		if (inside) {
			f32x4_t v[PT + TAPS - 1], w[TAPS];
#pragma unroll
			for (int i = 0; i < TAPS; i++) w[i] = tg_load4(d.conv + (size_t)i * d.channels + c);
#pragma unroll
			for (int i = 0; i < PT + TAPS - 1; i++) v[i] = tg_load4(x + (size_t)(t0 - TAPS + 1 + i) * ld + c);
#pragma unroll
			for (int i = 0; i < TAPS; i++)
#pragma unroll
				for (int p = 0; p < PT; p++)
#pragma unroll
					for (int e = 0; e < 4; e++) r[p][e] = fmaf(w[i][e], v[p + i][e], r[p][e]);
		}
	}
	for (int i = 0; i < (inside ? 0 : d.taps); i++) {
		const f32x4_t w = tg_load4(d.conv + (size_t)i * d.channels + c);
#pragma unroll
		for (int p = 0; p < PT; p++) {
			const int from = min(t0 + p, n - 1) - d.taps + 1 + i;
			f32x4_t v = {0, 0, 0, 0};
			if (from >= 0) v = tg_load4(x + (size_t)from * ld + c);
			else if (past + from >= 0) v = tg_load4(d.ring + (size_t)((past + from) % d.taps) * d.channels + c);
#pragma unroll
			for (int e = 0; e < 4; e++) r[p][e] = fmaf(w[e], v[e], r[p][e]);
		}
	}
#pragma unroll
	for (int p = 0; p < PT; p++) {
		float ss = 0.0f, f = 1.0f;
#pragma unroll
		for (int e = 0; e < 4; e++) {
			r[p][e] = tg_silu(r[p][e]);
			ss = fmaf(r[p][e], r[p][e], ss);
		}
		if (head) f = 1.0f / sqrtf(tg_wave_sum(in ? ss : 0.0f) + 1e-6f);
#pragma unroll
		for (int e = 0; e < 4; e++) r[p][e] *= f;
		if (in && t0 + p < n) tg_store4(head ? qk + (size_t)(t0 + p) * 2 * qc + c : v_out + (size_t)(t0 + p) * (d.channels - 2 * qc) + c - 2 * qc, r[p]);
	}
}

// ---- the pass over the chunks: 16 value columns of a head per workgroup --------------------------------------------------------
// Wave w keeps rows 16 (w + 4 i) ... of S in accumulators, which are the second operand of the products with the solved keys as
// they are; the waves' parts of those products meet in LDS, and u, again in accumulator layout, is the second operand of S's
// update.  The last inputs of the convolution go to the ring on the way.
// AHEAD: chunks whose operands are in registers or on their way.  The chunks are padded to a multiple of it (scratch too), with
// steps that leave S as it is: a branch around a chunk would make every wait cover all loads in flight.
constexpr int SCAN_AHEAD = 3;
template <class TR, int ND, int AHEAD>
__global__ __launch_bounds__(256, 1) void delta_scan_kernel(TgDelta d, const typename TR::T *x, int ld, int n, int past, const float *b, float *u,
                                                         const float *wk, const float *kt, float *st, int chunks) {
	__shared__ __align__(16) f32x4_t s_p[4][4][64], s_u[4][64];
	const TgGla &g = d.g;
	const int h = blockIdx.x, v0 = blockIdx.y * 16, tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lg = lane >> 4;
	const int hd = g.heads * g.dimp, ntile = g.dimp / 16;
	{
		const int keep = min(d.taps, n), total = keep * d.channels, step = (int)(gridDim.x * gridDim.y) * 256;
		for (int e = ((int)blockIdx.y * (int)gridDim.x + h) * 256 + tid; e < total; e += step) {
			const int i = e / d.channels, c = e - i * d.channels, t = n - keep + i;
			d.ring[(size_t)((past + t) % d.taps) * d.channels + c] = (float)x[(size_t)t * ld + c];
		}
	}
	f32x4_t S[ND];
	f32x4_t fw[AHEAD][ND][4], fk[AHEAD][ND][4], fb[AHEAD][ND], fv[AHEAD];
	bool own[ND];
	int row[ND];  // first row of the tile (the last tile again where there is none; its part counts as zero)
#pragma unroll
	for (int i = 0; i < ND; i++) {
		own[i] = w + 4 * i < ntile;
		row[i] = 16 * min(w + 4 * i, ntile - 1);
#pragma unroll
		for (int e = 0; e < 4; e++) S[i][e] = own[i] ? g.state[((size_t)h * g.dimp + row[i] + 4 * lg + e) * g.vdimp + v0 + lr] : 0.0f;
	}
	const int vt = (int)blockIdx.y, vtiles = g.vdimp / 16;
	const unsigned l4 = (unsigned)(lane * 4);
	// (bases that the workgroup shares, 32-bit offsets per lane)
	auto keys = [&](int ch) { return ((size_t)min(ch, chunks - 1) * g.heads + h) * g.dimp * C; };
	auto values = [&](int ch) { return (((size_t)ch * g.heads + h) * vtiles + vt) * 1024; };
	auto fetch_w = [&](int set, int ch) {
		const float *pw = wk + keys(ch), *pb = b + ((size_t)min(ch, chunks - 1) * C + C - 1) * hd + (size_t)h * g.dimp;
#pragma unroll
		for (int i = 0; i < ND; i++) {
#pragma unroll
			for (int tt = 0; tt < 4; tt++) fw[set][i][tt] = tg_load4(pw + (unsigned)(row[i] * C + tt * 256) + l4);
			fb[set][i] = tg_load4(pb + (unsigned)(row[i] + 4 * lg));
		}
		fv[set] = tg_load4(u + values(min(ch, chunks - 1)) + (unsigned)(w * 256) + l4);
	};
	auto fetch_k = [&](int set, int ch) {
		const float *pk = kt + keys(ch);
#pragma unroll
		for (int i = 0; i < ND; i++)
#pragma unroll
			for (int tt = 0; tt < 4; tt++) fk[set][i][tt] = tg_load4(pk + (unsigned)(row[i] * C + tt * 256) + l4);
	};
	// A wave issues in order and a load takes its time to issue: loads are dealt out among the matrix instructions of the two
	// products, each set's as soon as it has been used (past the end: the last chunk again, unused).
	auto chunk = [&](int set, int ch) {
		const bool live = ch < chunks;
		f32x4_t part[4];
#pragma unroll
		for (int tt = 0; tt < 4; tt++) part[tt] = f32x4_t{0, 0, 0, 0};
		fetch_k((set + AHEAD - 1) % AHEAD, ch + AHEAD - 1);
#pragma unroll
		for (int i = 0; i < ND; i++)
#pragma unroll
			for (int e = 0; e < 4; e++)
#pragma unroll
				for (int tt = 0; tt < 4; tt++) part[tt] = __builtin_amdgcn_mfma_f32_16x16x4f32(fw[set][i][tt][e], S[i][e], part[tt], 0, 0, 0);
#pragma unroll
		for (int i = 0; i < 4 * ND; i++) {
			__builtin_amdgcn_sched_group_barrier(0x008, 4, 0);  // matrix instructions
			__builtin_amdgcn_sched_group_barrier(0x020, 1, 0);  // global load
		}
		__builtin_amdgcn_sched_barrier(0);
#pragma unroll
		for (int tt = 0; tt < 4; tt++) s_p[w][tt][lane] = part[tt];
		// (a tile that is not there is written behind the last chunk: no branches, as above)
#pragma unroll
		for (int i = 0; i < ND; i++) {
			float *front = st + values(own[i] ? ch : chunks + AHEAD - 1) / C * g.dimp;
			tg_store4(front + (unsigned)(row[i] * 16) + l4, S[i]);
		}
		f32x4_t uv = fv[set];
#pragma unroll
		for (int i = 0; i < ND; i++)
#pragma unroll
			for (int e = 0; e < 4; e++) S[i][e] *= live ? pow2(fb[set][i][e]) : 1.0f;
		tg_lds_barrier();
		f32x4_t pq[4];
#pragma unroll
		for (int q = 0; q < 4; q++) pq[q] = s_p[q][w][lane];
#pragma unroll
		for (int e = 0; e < 4; e++) uv[e] = live ? uv[e] - ((pq[0][e] + pq[1][e]) + (pq[2][e] + pq[3][e])) : 0.0f;
		s_u[w][lane] = uv;
		tg_store4(u + values(ch) + (unsigned)(w * 256) + l4, uv);
		tg_lds_barrier();
		f32x4_t ut[4];
#pragma unroll
		for (int tt = 0; tt < 4; tt++) ut[tt] = s_u[tt][lane];
		__builtin_amdgcn_sched_barrier(0);
		fetch_w(set, ch + AHEAD);
#pragma unroll
		for (int tt = 0; tt < 4; tt++)
#pragma unroll
			for (int e = 0; e < 4; e++)
#pragma unroll
				for (int i = 0; i < ND; i++) S[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(fk[set][i][tt][e], ut[tt][e], S[i], 0, 0, 0);
#pragma unroll
		for (int i = 0; i < 5 * ND + 1; i++) {
			__builtin_amdgcn_sched_group_barrier(0x008, 3, 0);
			__builtin_amdgcn_sched_group_barrier(0x020, 1, 0);
		}
		__builtin_amdgcn_sched_barrier(0);
#pragma unroll
		for (int i = 0; i < ND; i++)
#pragma unroll
			for (int e = 0; e < 4; e++) S[i][e] = own[i] ? S[i][e] : 0.0f;
	};
#pragma unroll
	for (int a = 0; a < AHEAD; a++) {
		fetch_w(a, a);
		if (a + 1 < AHEAD) fetch_k(a, a);
		__builtin_amdgcn_sched_barrier(0);
	}
	for (int ch = 0; ch < chunks; ch += AHEAD) {
#pragma unroll
		for (int a = 0; a < AHEAD; a++) {
			chunk(a, ch + a);
			__builtin_amdgcn_sched_barrier(0);
		}
	}
#pragma unroll
	for (int i = 0; i < ND; i++)
		if (own[i])
#pragma unroll
			for (int e = 0; e < 4; e++) g.state[((size_t)h * g.dimp + row[i] + 4 * lg + e) * g.vdimp + v0 + lr] = S[i][e];
}

// ---- one token: 32 value columns of a head per workgroup, lane = 4 columns, 32 groups of key channels (R rows of S per lane) ------
template <int R>
__global__ __launch_bounds__(256) void delta_step_kernel(const float *y, TgDelta d, int g_off, int b_off, int a_off, const int *ctr, int host_pos,
                                                         float *o, float *gate) {
	constexpr int DM = 32 * R;
	__shared__ __align__(16) float s_q[DM], s_k[DM], s_a[DM], s_z[DM > 256 ? DM : 256], s_v[32], s_g[8][32];
	__shared__ f32x4_t s_rp[4][8], s_rq[4][8];
	__shared__ float s_sum[3][4];
	const TgGla &g = d.g;
	const int h = blockIdx.x, kh = h / g.group, c0 = blockIdx.y * 32, tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
	const int col = c0 + (tid & 7) * 4, dg = tid >> 3, hd = g.heads * g.dimp, hv = g.heads * g.vdimp, qc = d.q_channels();
	const int pos = host_pos >= 0 ? host_pos : ctr[0];
	float *S = g.state + ((size_t)h * g.dimp) * g.vdimp + col;
	f32x4_t st[R];
#pragma unroll
	for (int r = 0; r < R; r++) st[r] = tg_load4(S + (size_t)min(dg + 32 * r, g.dimp - 1) * g.vdimp);
	const float step = y[b_off + h];
	// Everything is requested before anything is used or stored: the convolution's inputs (CT earlier ones per round) of a key or
	// query channel and of a value channel, the decay's and the gate's low-rank products.
	constexpr int CT = 4, RA = 16, RG = 8;
	const int slot = pos % d.taps, ch_v = 2 * qc + h * g.vdimp + c0 + (tid & 31);
	struct Conv {
		float x, wx, w[CT], in[CT];
	};
	auto conv_request = [&](int c, int i0, Conv &r) {  // earlier inputs i0 ... i0 + CT - 1, oldest first (zero before the start)
		r.x = y[c];
		r.wx = d.conv[(size_t)(d.taps - 1) * d.channels + c];
#pragma unroll
		for (int i = 0; i < CT; i++) {
			const int at = min(i0 + i, d.taps - 1), from = slot + 1 + at;  // row of position pos - taps + 1 + at
			r.w[i] = d.conv[(size_t)at * d.channels + c];
			r.in[i] = d.ring[(size_t)(from >= d.taps ? from - d.taps : from) * d.channels + c];
		}
	};
	auto conv_sum = [&](int c, Conv &r) {
		float v = 0.0f;
		for (int i0 = 0; i0 < d.taps - 1; i0 += CT) {
			if (i0) conv_request(c, i0, r);
#pragma unroll
			for (int i = 0; i < CT; i++) v = i0 + i < d.taps - 1 ? fmaf(r.w[i], r.in[i], v) : v;
		}
		return tg_silu(fmaf(r.x, r.wx, v));
	};
	auto qk_channel = [&](int e) { return (e >= g.dimp ? qc - g.dimp : 0) + kh * g.dimp + e; };
	const int ns = g.dimp >= 256 ? 1 : 256 / g.dimp, per = (g.rank + ns - 1) / ns;  // the rank split over the lanes that the channels leave
	float wa[RA], ya[RA], wg[RG], yg[RG];
	auto decay_request = [&](int e, int j0) {
		const int sp = e / g.dimp, c = h * g.dimp + e - sp * g.dimp;
#pragma unroll
		for (int j = 0; j < RA; j++) {
			const int at = min(sp * per + j0 + j, g.rank - 1);
			wa[j] = g.a2[(size_t)at * hd + c];
			ya[j] = y[a_off + at];
		}
	};
	const int gp = (d.gate_rank + 7) / 8, glo = (tid >> 5) * gp, cg = h * g.vdimp + c0 + (tid & 31);
	auto gate_request = [&](int j0) {
#pragma unroll
		for (int j = 0; j < RG; j++) {
			const int at = min(glo + j0 + j, d.gate_rank - 1);
			wg[j] = d.g2[(size_t)at * hv + cg];
			yg[j] = y[g_off + at];
		}
	};
	Conv ck, cv;
	conv_request(qk_channel(min(tid, 2 * g.dimp - 1)), 0, ck);
	conv_request(ch_v, 0, cv);
	decay_request(min(tid, ns * g.dimp - 1), 0);
	gate_request(0);
	const float rate = expf(g.a_log[h]);

	const bool keep_qk = h % g.group == 0 && blockIdx.y == 0;  // the workgroup that keeps the newest input of these channels
	for (int e = tid; e < 2 * g.dimp; e += 256) {
		if (e != tid) conv_request(qk_channel(e), 0, ck);
		const float v = conv_sum(qk_channel(e), ck);
		(e >= g.dimp ? s_k[e - g.dimp] : s_q[e]) = v;
		if (keep_qk) d.ring[(size_t)slot * d.channels + qk_channel(e)] = ck.x;
	}
	{
		const float v = conv_sum(ch_v, cv);
		if (tid < 32) {
			s_v[tid] = v;
			d.ring[(size_t)slot * d.channels + ch_v] = cv.x;
		}
	}
	for (int e = tid; e < ns * g.dimp; e += 256) {
		const int lo = e / g.dimp * per, cnt = min(g.rank - lo, per);
		float z = 0.0f;
		for (int j0 = 0; j0 < cnt; j0 += RA) {
			if (e != tid || j0) decay_request(e, j0);
#pragma unroll
			for (int j = 0; j < RA; j++) z = j0 + j < cnt ? fmaf(wa[j], ya[j], z) : z;
		}
		s_z[e] = z;
	}
	{
		const int cnt = min(d.gate_rank - glo, gp);
		float z = 0.0f;
		for (int j0 = 0; j0 < cnt; j0 += RG) {
			if (j0) gate_request(j0);
#pragma unroll
			for (int j = 0; j < RG; j++) z = j0 + j < cnt ? fmaf(wg[j], yg[j], z) : z;
		}
		s_g[tid >> 5][tid & 31] = z;
	}
	__syncthreads();
	float sq = 0.0f, sk = 0.0f, skq = 0.0f;
	for (int c = tid; c < g.dimp; c += 256) {
		const float q = s_q[c], k = s_k[c];
		sq = fmaf(q, q, sq);
		sk = fmaf(k, k, sk);
		skq = fmaf(q, k, skq);
		float z = g.a2b[h * g.dimp + c];
		for (int sp = 0; sp < ns; sp++) z += s_z[sp * g.dimp + c];
		s_a[c] = pow2(tg_log2_sigmoid(-z) * rate);
	}
	sq = tg_wave_sum(sq);
	sk = tg_wave_sum(sk);
	skq = tg_wave_sum(skq);
	if (lane == 0) {
		s_sum[0][w] = sq;
		s_sum[1][w] = sk;
		s_sum[2][w] = skq;
	}
	if (tid < 32) {
		float z = 0.0f;
#pragma unroll
		for (int i = 0; i < 8; i++) z += s_g[i][tid];
		gate[h * g.vdimp + c0 + tid] = z;
	}
	__syncthreads();
	auto sum4 = [&](int i) { return (s_sum[i][0] + s_sum[i][1]) + (s_sum[i][2] + s_sum[i][3]); };
	const float fq = g.qscale / sqrtf(sum4(0) + 1e-6f), fk = 1.0f / sqrtf(sum4(1) + 1e-6f), kq = sum4(2) * fk * fq;
	f32x4_t ap = {0, 0, 0, 0}, aq = {0, 0, 0, 0};
	float kr[R];
#pragma unroll
	for (int r = 0; r < R; r++) {
		const int c = dg + 32 * r;
		const bool in = c < g.dimp;
		const int cc = in ? c : 0;
		const float a = s_a[cc], q = in ? s_q[cc] * fq : 0.0f;
		kr[r] = in ? s_k[cc] * fk : 0.0f;
#pragma unroll
		for (int e = 0; e < 4; e++) {
			st[r][e] *= a;
			ap[e] = fmaf(st[r][e], kr[r], ap[e]);
			aq[e] = fmaf(st[r][e], q, aq[e]);
		}
	}
#pragma unroll
	for (int e = 0; e < 4; e++) {
		ap[e] += tg_red_partner<32>(ap[e]);
		ap[e] += tg_red_partner<16>(ap[e]);
		ap[e] += tg_red_partner<8>(ap[e]);
		aq[e] += tg_red_partner<32>(aq[e]);
		aq[e] += tg_red_partner<16>(aq[e]);
		aq[e] += tg_red_partner<8>(aq[e]);
	}
	if (lane < 8) {
		s_rp[w][lane] = ap;
		s_rq[w][lane] = aq;
	}
	__syncthreads();
	const float beta = tg_sigmoid(step);
	f32x4_t u, r0;
#pragma unroll
	for (int e = 0; e < 4; e++) {
		const int i = tid & 7;
		u[e] = beta * (s_v[i * 4 + e] - ((s_rp[0][i][e] + s_rp[1][i][e]) + (s_rp[2][i][e] + s_rp[3][i][e])));
		r0[e] = fmaf(kq, u[e], (s_rq[0][i][e] + s_rq[1][i][e]) + (s_rq[2][i][e] + s_rq[3][i][e]));
	}
#pragma unroll
	for (int r = 0; r < R; r++) {
		const int c = dg + 32 * r;
		if (c < g.dimp) {
#pragma unroll
			for (int e = 0; e < 4; e++) st[r][e] = fmaf(kr[r], u[e], st[r][e]);
			tg_store4(S + (size_t)c * g.vdimp, st[r]);
		}
	}
	if (tid < 8) tg_store4(o + (size_t)h * g.vdimp + col, r0);
}

template <class TR>
void launch_delta_rows(const TgDelta &d, const void *xv, int ld, const float *low, int ld_low, int b_off, int a_off, const void *gate, int ldg, int n,
                       int past, const TgDeltaScratch &t, void *out, int ld_out, hipStream_t s) {
	const typename TR::T *x = (const typename TR::T *)xv;
	const TgGla &g = d.g;
	const int qc = d.q_channels(), hv = g.heads * g.vdimp, hd = g.heads * g.dimp, kvh = g.heads / g.group;
	const unsigned chunks = (unsigned)((n + C - 1) / C);
	auto prep = [&](auto *kernel) {
		hipLaunchKernelGGL(kernel, dim3((unsigned)((n + 4 * PT - 1) / (4 * PT)), (unsigned)(2 * kvh + (hv + 255) / 256)), dim3(256), 0, s, d, x, ld, n, past,
		                   t.qk, t.v);
	};
	if (d.taps == 4) prep(delta_prep_kernel<TR, 4>);
	else if (d.taps == 3) prep(delta_prep_kernel<TR, 3>);
	else prep(delta_prep_kernel<TR, 0>);
	hipLaunchKernelGGL(gla_decay_kernel, dim3(chunks, (unsigned)((hd + 63) / 64)), dim3(256), 0, s, low + a_off, ld_low, g, n, t.b);
	hipLaunchKernelGGL((gla_intra_kernel<TgF32, true>), dim3(chunks, (unsigned)g.heads), dim3(256), 0, s, t.qk, 2 * qc, qc, g, n, t.b, t.a,
	                   DeltaIntra{low + b_off, ld_low, t.t});
	const DeltaSolve solve = {t.qk, t.b, t.t, low + b_off, 2 * qc, qc, ld_low, t.v, t.u, t.wk, t.kt};
	hipLaunchKernelGGL(delta_solve_kernel, dim3(chunks, (unsigned)g.heads, (unsigned)((g.dimp + g.vdimp + 127) / 128)), dim3(256), 0, s, solve, g, n);
	const dim3 grid((unsigned)g.heads, (unsigned)(g.vdimp / 16));
	auto scan = [&](auto *kernel) {
		hipLaunchKernelGGL(kernel, grid, dim3(256), 0, s, d, x, ld, n, past, (const float *)t.b, t.u, (const float *)t.wk, (const float *)t.kt, t.st,
		                   (int)chunks);
	};
	if (g.dimp <= 64) scan(delta_scan_kernel<TR, 1, SCAN_AHEAD>);
	else if (g.dimp <= 128) scan(delta_scan_kernel<TR, 2, SCAN_AHEAD>);
	else scan(delta_scan_kernel<TR, 4, 2>);
	launch_out<TgF32, TR, true>(g, OutIn{t.qk, t.u, gate, 2 * qc, 0, ldg}, n, t.b, t.a, t.st, out, ld_out, s);
}

}  // namespace

void tg_launch_gla_step(const TgGla &g, const float *y, int k_off, int v_off, int a_off, float *o, hipStream_t s) {
	hipLaunchKernelGGL(gla_step_kernel, dim3((unsigned)g.heads, (unsigned)(g.vdimp / 32)), dim3(256), sizeof(float) * 3 * (size_t)g.dimp, s, y, g,
	                   k_off, v_off, a_off, o);
}

size_t tg_gla_scratch(const TgGla &g, int n, TgGlaScratch *t, unsigned char *base) {
	const size_t chunks = (size_t)((n + C - 1) / C), hd = (size_t)g.heads * g.dimp;
	size_t off = 0;
	auto take = [&](float **p, size_t floats) {
		if (base) *p = (float *)(base + off);
		off += (floats * sizeof(float) + 255) / 256 * 256;
	};
	TgGlaScratch tmp;
	if (!t) t = &tmp;
	take(&t->b, chunks * C * hd);
	take(&t->a, chunks * g.heads * C * C);
	take(&t->u, chunks * hd * g.vdimp);
	return off;
}

void tg_launch_gla_rows(const TgGla &g, int dt, const void *qkv, int ld, int k_off, int v_off, int g_off, const float *low, int ld_low, int n,
                        const TgGlaScratch &t, void *out, int ld_out, hipStream_t s) {
	if (dt == TG_DT_BF16) launch_rows<TgB16>(g, qkv, ld, k_off, v_off, g_off, low, ld_low, n, t, out, ld_out, s);
	else launch_rows<TgF32>(g, qkv, ld, k_off, v_off, g_off, low, ld_low, n, t, out, ld_out, s);
}

void tg_launch_delta_step(const TgDelta &d, const float *y, int g_off, int b_off, int a_off, const int *ctr, int host_pos, float *o, float *gate,
                          hipStream_t s) {
	const dim3 grid((unsigned)d.g.heads, (unsigned)(d.g.vdimp / 32));
	auto go = [&](auto *kernel) { hipLaunchKernelGGL(kernel, grid, dim3(256), 0, s, y, d, g_off, b_off, a_off, ctr, host_pos, o, gate); };
	if (d.g.dimp <= 64) go(delta_step_kernel<2>);
	else if (d.g.dimp <= 128) go(delta_step_kernel<4>);
	else go(delta_step_kernel<8>);
}

size_t tg_delta_scratch(const TgDelta &d, int n, TgDeltaScratch *t, unsigned char *base) {
	const TgGla &g = d.g;
	const size_t chunks = (size_t)((n + C - 1) / C), hd = (size_t)g.heads * g.dimp, hv = (size_t)g.heads * g.vdimp;
	const size_t padded = chunks + SCAN_AHEAD;  // (what the pass over the chunks writes)
	size_t off = 0;
	auto take = [&](float **p, size_t floats) {
		if (base) *p = (float *)(base + off);
		off += (floats * sizeof(float) + 255) / 256 * 256;
	};
	TgDeltaScratch tmp;
	if (!t) t = &tmp;
	take(&t->b, chunks * C * hd);
	take(&t->a, chunks * g.heads * C * C);
	take(&t->t, chunks * g.heads * C * C);
	take(&t->qk, (size_t)n * 2 * d.q_channels());
	take(&t->v, (size_t)n * hv);
	take(&t->u, padded * C * hv);
	take(&t->wk, chunks * C * hd);
	take(&t->kt, chunks * C * hd);
	take(&t->st, padded * hd * g.vdimp);
	return off;
}

void tg_launch_delta_rows(const TgDelta &d, int dt, const void *x, int ld, const float *low, int ld_low, int b_off, int a_off, const void *gate, int ldg,
                          int n, int past, const TgDeltaScratch &t, void *out, int ld_out, hipStream_t s) {
	if (dt == TG_DT_BF16) launch_delta_rows<TgB16>(d, x, ld, low, ld_low, b_off, a_off, gate, ldg, n, past, t, out, ld_out, s);
	else launch_delta_rows<TgF32>(d, x, ld, low, ld_low, b_off, a_off, gate, ldg, n, past, t, out, ld_out, s);
}
