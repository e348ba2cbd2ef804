// Gated linear attention: the step of one token, and the chunked form of many (tg_gla.h).
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
	const float bias = g.a2b[cc];
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
		if (real && t0 + 16 * w + i < n) run += tg_log2_sigmoid(z[i]) * g.inv_tau;  // past the end: the sum stays
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

template <class TR>
__global__ __launch_bounds__(256) void gla_intra_kernel(const typename TR::T *qkv, int ld, int k_off, TgGla g, int n, const float *b, float *A) {
	__shared__ __align__(16) float s_q[C][SLP], s_k[C][SLP], s_b[C][SLP];
	const int ch = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
	const int lr = lane & 15, lg = lane >> 4, hd = g.heads * g.dimp, t0 = ch * C;
	f32x4_t off[3], dia = {0, 0, 0, 0};
#pragma unroll
	for (int j = 0; j < 3; j++) off[j] = f32x4_t{0, 0, 0, 0};
	for (int d0 = 0; d0 < g.dimp; d0 += SL) {
		__syncthreads();
		for (int e = tid; e < C * SL / 4; e += 256) {
			const int r = e / (SL / 4), c4 = (e % (SL / 4)) * 4, t = t0 + r;
			const size_t col = (size_t)h * g.dimp + d0 + c4;
			f32x4_t q = tg_load4(qkv + (size_t)min(t, n - 1) * ld + col), k = tg_load4(qkv + (size_t)min(t, n - 1) * ld + k_off + col);
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
				const float qv = s_q[qi][d] * pow2(s_b[qi][d] - ref);
#pragma unroll
				for (int j = 0; j < 3; j++)
					if (j < w) {
						const float kv = s_k[16 * j + lr][d] * pow2(ref - s_b[16 * j + lr][d]);
						off[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(qv, kv, off[j], 0, 0, 0);
					}
			}
		}
		for (int d = 0; d < SL; d += 4) {
			const f32x4_t q = tg_load4(&s_q[qi][d]), bi = tg_load4(&s_b[qi][d]);
#pragma unroll
			for (int j = 0; j < 4; j++) {
				const int kj = 16 * w + 4 * lg + j;
				const f32x4_t k = tg_load4(&s_k[kj][d]), bj = tg_load4(&s_b[kj][d]);
				if (kj <= qi) {
#pragma unroll
					for (int e = 0; e < 4; e++) dia[j] = fmaf(q[e] * k[e], pow2(bi[e] - bj[e]), dia[j]);
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
template <class TR, int VB>
__global__ __launch_bounds__(512) void gla_out_kernel(const typename TR::T *qkv, int ld, int v_off, int g_off, TgGla g, int n, const float *b,
                                                      const float *A, const float *U, typename TR::T *out, int ld_out) {
	constexpr int XP = 36, YP = VB + 16, NI = VB / 32, NY = 32 * VB / 4 / 512;
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
			x = tg_load4(qkv + (size_t)min(t0 + xr, n - 1) * ld + qc);
			bx = tg_load4(b + (size_t)(t0 + xr) * hd + qc);
#pragma unroll
			for (int i = 0; i < NY; i++) {
				const int e = tid + 512 * i, r = e / (VB / 4), c4 = (e % (VB / 4)) * 4;
				y[i] = tg_load4(S + (size_t)(sl * 32 + r) * g.vdimp + (c4 < g.vdimp ? c4 : 0));
			}
		} else {
			const int j0 = (sl - slabs) * 32;
			x = tg_load4(A + (((size_t)ch * g.heads + h) * C + xr) * C + j0 + xc);
#pragma unroll
			for (int i = 0; i < NY; i++) {
				const int e = tid + 512 * i, r = e / (VB / 4), c4 = (e % (VB / 4)) * 4;
				y[i] = tg_load4(qkv + (size_t)min(t0 + j0 + r, n - 1) * ld + v_off + (size_t)h * g.vdimp + (c4 < g.vdimp ? c4 : 0));
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
			tg_store4(&s_y[r][c4], c4 < g.vdimp ? y[i] : f32x4_t{0, 0, 0, 0});  // (rows of v past the end meet zeros of A)
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
	const typename TR::T *gate = qkv + (size_t)t * ld + g_off + (size_t)h * g.vdimp;
#pragma unroll
	for (int j = 0; j < NI; j++) {
		const int v = wv + 16 * j + 4 * lg;
		if (v < g.vdimp) {
			const f32x4_t gv = tg_load4(gate + v), nw = tg_load4(g.norm + v);
			f32x4_t r;
#pragma unroll
			for (int e = 0; e < 4; e++) r[e] = acc[j][e] * inv * nw[e] * tg_silu(gv[e]);
			tg_store4(dst + v, r);
		}
	}
	if (h == g.heads - 1)  // the columns behind the heads
		for (int v = g.heads * g.vdimp + (w >> 2) * 16 + 4 * lg; v < ld_out; v += 32) tg_store4(out + (size_t)t * ld_out + v, f32x4_t{0, 0, 0, 0});
}

template <class TR, int VB>
void launch_out(const TgGla &g, const typename TR::T *x, int ld, int v_off, int g_off, int n, const TgGlaScratch &t, typename TR::T *out, int ld_out,
                hipStream_t s) {
	hipLaunchKernelGGL((gla_out_kernel<TR, VB>), dim3((unsigned)((n + C - 1) / C), (unsigned)g.heads), dim3(512), 0, s, x, ld, v_off, g_off, g, n, t.b,
	                   t.a, t.u, out, ld_out);
}

template <class TR>
void launch_rows(const TgGla &g, const void *qkv, int ld, int k_off, int v_off, int g_off, const float *low, int ld_low, int n,
                 const TgGlaScratch &t, void *out, int ld_out, hipStream_t s) {
	typedef typename TR::T T;
	const T *x = (const T *)qkv;
	T *o = (T *)out;
	const unsigned chunks = (unsigned)((n + C - 1) / C), H = (unsigned)g.heads, hd = (unsigned)(g.heads * g.dimp), nd = (unsigned)((g.dimp + 127) / 128);
	hipLaunchKernelGGL(gla_decay_kernel, dim3(chunks, (hd + 63) / 64), dim3(256), 0, s, low, ld_low, g, n, t.b);
	hipLaunchKernelGGL((gla_intra_kernel<TR>), dim3(chunks, H), dim3(256), 0, s, x, ld, k_off, g, n, t.b, t.a);
	if (g.vdimp <= 64)
		hipLaunchKernelGGL((gla_state_kernel<TR, 64>), dim3(chunks, H, nd), dim3(512), 0, s, x, ld, k_off, v_off, g, n, t.b, t.u);
	else
		hipLaunchKernelGGL((gla_state_kernel<TR, 128>), dim3(chunks, H, nd * (unsigned)((g.vdimp + 127) / 128)), dim3(512), 0, s, x, ld, k_off, v_off, g,
		                   n, t.b, t.u);
	const size_t per = (size_t)hd * g.vdimp;
	hipLaunchKernelGGL(gla_scan_kernel, dim3((unsigned)((per + 255) / 256)), dim3(256), 0, s, t.u, t.b, g, (int)chunks);
	if (g.vdimp <= 64) launch_out<TR, 64>(g, x, ld, v_off, g_off, n, t, o, ld_out, s);
	else if (g.vdimp <= 128) launch_out<TR, 128>(g, x, ld, v_off, g_off, n, t, o, ld_out, s);
	else if (g.vdimp <= 256) launch_out<TR, 256>(g, x, ld, v_off, g_off, n, t, o, ld_out, s);
	else launch_out<TR, TG_GLA_VDIM_MAX>(g, x, ld, v_off, g_off, n, t, o, ld_out, s);
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
