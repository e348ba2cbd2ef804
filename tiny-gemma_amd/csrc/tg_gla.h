// Gated linear attention with a decay per key channel (tg_gla.hip).  Per head, with a [dim][vdim] state in fp32:
//     S_t = diag(alpha_t) S_(t-1) + k_t v_t^T,   o_t = S_t^T (q_t / sqrt(dim)),   alpha_t = sigmoid(z_t)^(1 / tau).
// Heads are laid out with padded sizes dimp, vdimp (multiples of 32), the padding is zero.
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
