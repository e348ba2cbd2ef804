// Gated linear attention with a decay per key channel (tg_gla.hip).  Per head, with a [dim][vdim] state in fp32:
//     S_t = diag(alpha_t) S_(t-1) + k_t v_t^T,   o_t = S_t^T (q_t / sqrt(dim)),   alpha_t = sigmoid(z_t)^(1 / tau).
// Heads are laid out with padded sizes dimp, vdimp (multiples of 32), the padding is zero.
//
// The gated delta rule, on the same state and chunks (tg_delta_*): with unit k and step size beta
//     u_t = beta_t (v_t - (diag(alpha_t) S_(t-1))^T k_t),   S_t = diag(alpha_t) S_(t-1) + k_t u_t^T,   o_t = S_t^T (q_t / sqrt(dim)),
// q, k and v behind a short causal convolution over time, alpha_t = exp(-exp(A_log) softplus(z_t)), several heads per q/k head,
// a sigmoid gate of low rank.
#pragma once

#include "tg_linear.h"

#define TG_GLA_CHUNK 64
#define TG_GLA_VDIM_MAX 512  // largest padded value size of the chunked form

struct TgGla {
	int heads, dim, dimp, vdim, vdimp, rank;
	float qscale, inv_tau, eps;
	const float *a2;      // decay projection, transposed: [rank][heads * dimp]
	const float *a2b;     // [heads * dimp]
	const float *norm;    // [vdim]
	float *state;         // [heads][dimp][vdimp]
	const float *a_log;   // [heads]; null: alpha = sigmoid(z)^inv_tau, else exp(-exp(a_log) softplus(z))
	int group;            // heads per q/k head
};
// one token: y = the fused product's outputs q | k | v | g | a1 (offsets in floats); o [heads * vdimp]
void tg_launch_gla_step(const TgGla &g, const float *y, int k_off, int v_off, int a_off, float *o, hipStream_t s);
// n tokens: qkv [n][ld] in the model's format (q at column 0, offsets in elements), low [n][ld_low] fp32 (the decay's low-rank input).
// Scratch: see tg_gla_scratch.  out [n][ld_out]: the normalised, gated heads.
struct TgGlaScratch {
	float *b;       // [chunks * 64][heads * dimp] running sums of log2 alpha inside a chunk
	float *a;       // [chunks][heads][64][64]
	float *u;       // [chunks][heads][dimp][vdimp]
};
size_t tg_gla_scratch(const TgGla &g, int n, TgGlaScratch *t, unsigned char *base);  // bytes; fills *t when base is not null
void tg_launch_gla_rows(const TgGla &g, int dt, const void *qkv, int ld, int k_off, int v_off, int g_off, const float *low, int ld_low, int n,
                        const TgGlaScratch &t, void *out, int ld_out, hipStream_t s);

#define TG_DELTA_DIM_MAX 256   // largest padded key size

struct TgDelta {
	TgGla g;              // g.norm, g.a2, g.a2b, g.a_log, g.state, g.rank (of the decay) as above
	int taps, channels;   // convolution; channels: q | k | v, q and k [heads / group][dimp], v [heads][vdimp]
	const float *conv;    // [taps][channels], the last row meets the newest input
	float *ring;          // [taps][channels] inputs of the last tokens: position p in row p % taps
	const float *g2;      // output gate: [gate_rank][heads * vdimp]
	int gate_rank;
	__host__ __device__ int q_channels() const { return g.heads / g.group * g.dimp; }
};
// one token at position host_pos (or ctr[0] where host_pos < 0): y = the fused product's outputs, q | k | v from column 0, the rest
// at the offsets; o, gate [heads * vdimp]: read-out, and the gate before its sigmoid
void tg_launch_delta_step(const TgDelta &d, const float *y, int g_off, int b_off, int a_off, const int *ctr, int host_pos, float *o, float *gate,
                          hipStream_t s);
// n tokens behind `past` earlier ones: x [n][ld] q | k | v in the model's format; low [n][ld_low] fp32: step sizes at b_off, the decay's
// low-rank input at a_off; gate [n][ldg] in the model's format, before its sigmoid; out [n][ld_out]: the normalised, gated heads
struct TgDeltaScratch {
	float *b;       // [chunks * 64][heads * dimp] running sums of log2 alpha inside a chunk
	float *a;       // [chunks][heads][64][64] q . k with the decay between them
	float *t;       // [chunks][heads][64][64] what the solve multiplies with (tg_gla.hip)
	float *qk;      // [n][q | k] behind convolution and unit norm
	float *v;       // [n][heads * vdimp] behind the convolution
	// in operand order (tg_gla.hip):
	float *u;       // [chunks][heads][vdimp x 64] v's solved form, then u
	float *wk;      // [chunks][heads][dimp x 64] solved keys
	float *kt;      // [chunks][heads][dimp x 64] keys decayed to the chunk's end
	float *st;      // [chunks][heads][vdimp x dimp] the state in front of every chunk
};
size_t tg_delta_scratch(const TgDelta &d, int n, TgDeltaScratch *t, unsigned char *base);
void tg_launch_delta_rows(const TgDelta &d, int dt, const void *x, int ld, const float *low, int ld_low, int b_off, int a_off, const void *gate, int ldg,
                          int n, int past, const TgDeltaScratch &t, void *out, int ld_out, hipStream_t s);
