// Gated linear attention: the step of one token, and the chunked form of many (tg_gla.h).
//
// Chunked form.  With b_t the sum of log alpha over the chunk's tokens up to and including t, a chunk of 64 tokens that
// starts from state S contributes
//     o_i = (q_i e^{b_i})^T S + sum_{j <= i} A_ij v_j,   A_ij = sum_d q_id k_jd e^{b_id - b_jd},
//     S'  = diag(e^{b_end}) S + sum_j (k_j e^{b_end - b_j}) v_j^T,
// all exponents <= 0, whatever the decay: A's blocks of 16 x 16 below the diagonal take the exponent apart at the row
// block's first token (both halves <= 0) and run on the fp32 matrix instructions, the diagonal blocks are summed pair by
// pair.  Four launches: b; A and the chunks' own state contributions U, all chunks at once; the states in front of every
// chunk, one pass over U; the outputs, all chunks at once.  Everything is fp32 (q, k, v are read in the model's format).

#include "tg_gla.h"

namespace {

constexpr int C = TG_GLA_CHUNK;

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
		s_a[d] = expf(tg_log_sigmoid(z + g.a2b[c]) * g.inv_tau);
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
		if (real && t0 + 16 * w + i < n) run += tg_log_sigmoid(z[i]) * g.inv_tau;  // past the end: the sum stays
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
				const float qv = s_q[qi][d] * expf(s_b[qi][d] - ref);
#pragma unroll
				for (int j = 0; j < 3; j++)
					if (j < w) {
						const float kv = s_k[16 * j + lr][d] * expf(ref - s_b[16 * j + lr][d]);
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
					for (int e = 0; e < 4; e++) dia[j] = fmaf(q[e] * k[e], expf(bi[e] - bj[e]), dia[j]);
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

// ---- U = sum_j (k_j e^{b_end - b_j}) v_j^T: 64 key channels x 64 value columns per workgroup ----------------------------------
constexpr int BP = 68;
template <class TR>
__global__ __launch_bounds__(256) void gla_state_kernel(const typename TR::T *qkv, int ld, int k_off, int v_off, TgGla g, int n, const float *b,
                                                        float *U) {
	__shared__ __align__(16) float s_k[C][BP], s_v[C][BP];
	const int ch = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
	const int nvb = (g.vdimp + 63) / 64, d0 = (int)(blockIdx.z / nvb) * 64, v0 = (int)(blockIdx.z % nvb) * 64;
	const int lr = lane & 15, lg = lane >> 4, hd = g.heads * g.dimp, t0 = ch * C;
	for (int e = tid; e < C * 16; e += 256) {
		const int r = e >> 4, c4 = (e & 15) * 4, t = t0 + r, tc = min(t, n - 1);
		const bool kin = t < n && d0 + c4 < g.dimp, vin = t < n && v0 + c4 < g.vdimp;
		const size_t kc = (size_t)h * g.dimp + (kin ? d0 + c4 : 0), vc = (size_t)h * g.vdimp + (vin ? v0 + c4 : 0);
		const f32x4_t k = tg_load4(qkv + (size_t)tc * ld + k_off + kc), v = tg_load4(qkv + (size_t)tc * ld + v_off + vc);
		const f32x4_t be = tg_load4(b + (size_t)(t0 + C - 1) * hd + kc), bj = tg_load4(b + (size_t)t * hd + kc);
		f32x4_t ks, vs;
#pragma unroll
		for (int i = 0; i < 4; i++) {
			ks[i] = kin ? k[i] * expf(be[i] - bj[i]) : 0.0f;
			vs[i] = vin ? v[i] : 0.0f;
		}
		tg_store4(&s_k[r][c4], ks);
		tg_store4(&s_v[r][c4], vs);
	}
	__syncthreads();
	f32x4_t acc[4];
#pragma unroll
	for (int j = 0; j < 4; j++) acc[j] = f32x4_t{0, 0, 0, 0};
#pragma unroll 4
	for (int t = 0; t < C; t += 4) {
		const float a = s_k[t + lg][16 * w + lr];
#pragma unroll
		for (int j = 0; j < 4; j++) acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, s_v[t + lg][16 * j + lr], acc[j], 0, 0, 0);
	}
	float *out = U + ((size_t)ch * g.heads + h) * g.dimp * g.vdimp;
#pragma unroll
	for (int j = 0; j < 4; j++)
#pragma unroll
		for (int e = 0; e < 4; e++) {
			const int d = d0 + 16 * w + 4 * lg + e, v = v0 + 16 * j + lr;
			if (d < g.dimp && v < g.vdimp) out[(size_t)d * g.vdimp + v] = acc[j][e];
		}
}

// ---- U becomes the state in front of its chunk; the state behind the last chunk goes to the sequence ---------------------------
__global__ __launch_bounds__(256) void gla_scan_kernel(float *U, const float *b, TgGla g, int chunks) {
	const size_t per = (size_t)g.heads * g.dimp * g.vdimp, e = ((size_t)blockIdx.x * 256 + threadIdx.x) * 4;
	if (e >= per) return;
	const int hd = g.heads * g.dimp, c = (int)(e / g.vdimp);
	f32x4_t s = tg_load4(g.state + e), nxt = tg_load4(U + e);
	float bn = b[(size_t)(C - 1) * hd + c];
	for (int ch = 0; ch < chunks; ch++) {
		const f32x4_t u = nxt;
		const float dec = expf(bn);
		if (ch + 1 < chunks) {
			nxt = tg_load4(U + (size_t)(ch + 1) * per + e);
			bn = b[(size_t)((ch + 1) * C + C - 1) * hd + c];
		}
		tg_store4(U + (size_t)ch * per + e, s);
#pragma unroll
		for (int i = 0; i < 4; i++) s[i] = fmaf(dec, s[i], u[i]);
	}
	tg_store4(g.state + e, s);
}

// ---- o = (q e^b)^T S + A v: 64 tokens x 64 value columns per workgroup -----------------------------------------------------------
template <class TR>
__global__ __launch_bounds__(256) void gla_out_kernel(const typename TR::T *qkv, int ld, int v_off, TgGla g, int n, const float *b, const float *A,
                                                      const float *U, float *o) {
	__shared__ __align__(16) float s_a[C][BP], s_b[C][BP];
	const int ch = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * 64, tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
	const int lr = lane & 15, lg = lane >> 4, hd = g.heads * g.dimp, t0 = ch * C;
	const float *S = U + ((size_t)ch * g.heads + h) * g.dimp * g.vdimp;
	f32x4_t acc[4];
#pragma unroll
	for (int j = 0; j < 4; j++) acc[j] = f32x4_t{0, 0, 0, 0};
	// slabs of 64: the key channels (rows q e^b, columns of S), last the chunk's own tokens (rows A, columns v)
	const int slabs = (g.dimp + 63) / 64;
	for (int sl = 0; sl <= slabs; sl++) {
		__syncthreads();
		for (int e = tid; e < C * 16; e += 256) {
			const int r = e >> 4, c4 = (e & 15) * 4;
			const bool vin = v0 + c4 < g.vdimp;
			f32x4_t x, y;
			if (sl < slabs) {
				const int t = t0 + r, d = sl * 64 + c4;
				const bool qin = t < n && d < g.dimp, sin = sl * 64 + r < g.dimp && vin;
				const size_t qc = (size_t)h * g.dimp + (qin ? d : 0);
				const f32x4_t q = tg_load4(qkv + (size_t)min(t, n - 1) * ld + qc), bq = tg_load4(b + (size_t)t * hd + qc);
				const f32x4_t sv = tg_load4(S + (size_t)(sin ? sl * 64 + r : 0) * g.vdimp + (sin ? v0 + c4 : 0));
#pragma unroll
				for (int i = 0; i < 4; i++) {
					x[i] = qin ? q[i] * g.qscale * expf(bq[i]) : 0.0f;
					y[i] = sin ? sv[i] : 0.0f;
				}
			} else {
				const int t = t0 + r;
				const bool in = t < n && vin;
				x = tg_load4(A + (((size_t)ch * g.heads + h) * C + r) * C + c4);
				const f32x4_t v = tg_load4(qkv + (size_t)min(t, n - 1) * ld + v_off + (size_t)h * g.vdimp + (vin ? v0 + c4 : 0));
#pragma unroll
				for (int i = 0; i < 4; i++) y[i] = in ? v[i] : 0.0f;
			}
			tg_store4(&s_a[r][c4], x);
			tg_store4(&s_b[r][c4], y);
		}
		__syncthreads();
#pragma unroll 4
		for (int d = 0; d < 64; d += 4) {
			const float a = s_a[16 * w + lr][d + lg];
#pragma unroll
			for (int j = 0; j < 4; j++) acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, s_b[d + lg][16 * j + lr], acc[j], 0, 0, 0);
		}
	}
#pragma unroll
	for (int j = 0; j < 4; j++)
#pragma unroll
		for (int e = 0; e < 4; e++) {
			const int t = t0 + 16 * w + 4 * lg + e, v = v0 + 16 * j + lr;
			if (t < n && v < g.vdimp) o[(size_t)t * g.heads * g.vdimp + (size_t)h * g.vdimp + v] = acc[j][e];
		}
}

// ---- every head over its root mean square, times the norm's weight and silu(gate); a wave per (token, head) ------------------------
template <class TR>
__global__ __launch_bounds__(256) void gla_norm_gate_kernel(const float *o, const typename TR::T *gate, int ld, TgGla g, int n, typename TR::T *out,
                                                            int ld_out) {
	const int row = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
	const int per = g.heads + 1;  // the last "head" of a token clears the columns behind the heads
	if (row >= n * per) return;
	const int t = row / per, h = row - t * per;
	typename TR::T *dst = out + (size_t)t * ld_out + (size_t)h * g.vdimp;
	if (h == g.heads) {
		for (int v = h * g.vdimp + lane; v < ld_out; v += 64) out[(size_t)t * ld_out + v] = (typename TR::T)0.0f;
		return;
	}
	const float *x = o + ((size_t)t * g.heads + h) * g.vdimp;
	float ss = 0.0f;
	for (int v = lane; v < g.vdim; v += 64) ss = fmaf(x[v], x[v], ss);
	ss = tg_wave_sum(ss);
	const float inv = 1.0f / sqrtf(ss / (float)g.vdim + g.eps);
	for (int v = lane; v < g.vdimp; v += 64) {
		const bool in = v < g.vdim;
		const int vc = in ? v : 0;
		const float r = x[vc] * inv * g.norm[vc] * tg_silu((float)gate[(size_t)t * ld + (size_t)h * g.vdimp + vc]);
		dst[v] = (typename TR::T)(in ? r : 0.0f);
	}
}

template <class TR>
void launch_rows(const TgGla &g, const void *qkv, int ld, int k_off, int v_off, int g_off, const float *low, int ld_low, int n,
                 const TgGlaScratch &t, void *out, int ld_out, hipStream_t s) {
	typedef typename TR::T T;
	const T *x = (const T *)qkv;
	const unsigned chunks = (unsigned)((n + C - 1) / C), H = (unsigned)g.heads, hd = (unsigned)(g.heads * g.dimp);
	const unsigned ndb = (unsigned)((g.dimp + 63) / 64), nvb = (unsigned)((g.vdimp + 63) / 64);
	hipLaunchKernelGGL(gla_decay_kernel, dim3(chunks, (hd + 63) / 64), dim3(256), 0, s, low, ld_low, g, n, t.b);
	hipLaunchKernelGGL((gla_intra_kernel<TR>), dim3(chunks, H), dim3(256), 0, s, x, ld, k_off, g, n, t.b, t.a);
	hipLaunchKernelGGL((gla_state_kernel<TR>), dim3(chunks, H, ndb * nvb), dim3(256), 0, s, x, ld, k_off, v_off, g, n, t.b, t.u);
	const size_t per = (size_t)hd * g.vdimp;
	hipLaunchKernelGGL(gla_scan_kernel, dim3((unsigned)((per / 4 + 255) / 256)), dim3(256), 0, s, t.u, t.b, g, (int)chunks);
	hipLaunchKernelGGL((gla_out_kernel<TR>), dim3(chunks, H, nvb), dim3(256), 0, s, x, ld, v_off, g, n, t.b, t.a, t.u, t.o);
	const long long rows = (long long)n * (g.heads + 1);
	hipLaunchKernelGGL((gla_norm_gate_kernel<TR>), dim3((unsigned)((rows + 3) / 4)), dim3(256), 0, s, t.o, x + g_off, ld, g, n, (T *)out, ld_out);
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
	take(&t->o, (size_t)n * g.heads * g.vdimp);
	return off;
}

void tg_launch_gla_rows(const TgGla &g, int dt, const void *qkv, int ld, int k_off, int v_off, int g_off, const float *low, int ld_low, int n,
                        const TgGlaScratch &t, void *out, int ld_out, hipStream_t s) {
	if (dt == TG_DT_BF16) launch_rows<TgB16>(g, qkv, ld, k_off, v_off, g_off, low, ld_low, n, t, out, ld_out, s);
	else launch_rows<TgF32>(g, qkv, ld, k_off, v_off, g_off, low, ld_low, n, t, out, ld_out, s);
}
