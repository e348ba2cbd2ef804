// Products with bfloat16 or float32 weights (tg_linear.hip): what the layer-list models (tg_net.hip) are built from.
// Nothing here is part of the C ABI.
//
// Number formats.  A model runs in one of two: TG_DT_BF16 (weights and matrix operands bfloat16, accumulation fp32) or
// TG_DT_F32 (everything fp32; the matrix cores' fp32 instructions round like fused multiply-adds).  Residual stream, norms,
// scores, routers and recurrent state are fp32 in both.
//
// Weight layout.  W [N][K] (applied as W x) is stored in matrix-operand fragments of 1 KiB,
//     P[n / 16][k / KF][lane][KV elements],   lane = n % 16 + 16 * ((k % KF) / KV),
// KV = elements in 16 bytes (8 or 4), KF = 4 * KV (32 or 16): lane l holds the 16 bytes it feeds to the matrix
// instruction (bf16: one 16x16x32; fp32: four 16x16x4, element i of the 16 bytes in the i-th), a wave reads a fragment
// as one contiguous KiB, and the same bytes serve the one-row products of a decode step and the tiled products of a
// prefill.  N is padded to 16, K to 64 (head blocks: 32) with zeros, so every buffer that receives a product holds
// zeros in its padding and may be a padded operand of the next one.
#pragma once

#include "tg_internal.h"

enum { TG_DT_BF16 = 0, TG_DT_F32 = 1 };
inline size_t tg_dt_bytes(int dt) { return dt == TG_DT_BF16 ? 2 : 4; }
inline int tg_up(int x, int m) { return (x + m - 1) / m * m; }

#if defined(__HIPCC__)
typedef float f32x4_t __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4_t __attribute__((ext_vector_type(4)));

struct TgB16 {
	typedef __bf16 T;
	typedef bf16x8_t Frag;
	static constexpr int DT = TG_DT_BF16, KV = 8, KF = 32;
	static __device__ __forceinline__ f32x4_t mma(Frag a, Frag b, f32x4_t c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }
};
struct TgF32 {
	typedef float T;
	typedef f32x4_t Frag;
	static constexpr int DT = TG_DT_F32, KV = 4, KF = 16;
	static __device__ __forceinline__ f32x4_t mma(Frag a, Frag b, f32x4_t c) {
#pragma unroll
		for (int i = 0; i < 4; i++) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[i], c, 0, 0, 0);
		return c;
	}
};
__device__ __forceinline__ float tg_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float tg_gelu(float z) { return 0.5f * z * (1.0f + erff(z * 0.70710678118654752440f)); }
__device__ __forceinline__ float tg_silu(float z) { return z / (1.0f + expf(-z)); }
// log2(sigmoid(z)) = min(z, 0) log2 e - log2(1 + e^-|z|); for a small second term its series, which keeps it exact to the last bits
__device__ __forceinline__ float tg_log2_sigmoid(float z) {
	const float L2E = 1.44269504088896340736f;
	const float x = __builtin_amdgcn_exp2f(-fabsf(z) * L2E);
	const float series = x * fmaf(x, fmaf(x, fmaf(x, fmaf(x, 0.2f, -0.25f), 1.0f / 3.0f), -0.5f), 1.0f) * L2E;
	return fminf(z, 0.0f) * L2E - (x < 0.0625f ? series : __builtin_amdgcn_logf(1.0f + x));
}
// four consecutive values as one store
__device__ __forceinline__ void tg_store4(float *p, f32x4_t v) { *reinterpret_cast<f32x4_t *>(p) = v; }
__device__ __forceinline__ void tg_store4(__bf16 *p, f32x4_t v) { *reinterpret_cast<bf16x4_t *>(p) = __builtin_convertvector(v, bf16x4_t); }
__device__ __forceinline__ f32x4_t tg_load4(const float *p) { return *reinterpret_cast<const f32x4_t *>(p); }
__device__ __forceinline__ f32x4_t tg_load4(const __bf16 *p) { return __builtin_convertvector(*reinterpret_cast<const bf16x4_t *>(p), f32x4_t); }
#endif

// A packed matrix (see above); n, k are the padded sizes.
struct TgMat {
	void *w = nullptr;
	int n = 0, k = 0;
};

// One source tensor into (part of) a packed matrix.  Destination row i (of `rows`) comes from source row
// (i / gp) * g + i % gp where i % gp < g, else it is zero; destination column j likewise through kg, kgp.  It goes to row
// (i / 16) * 16 * frag_step + frag_off * 16 + i % 16 of the matrix: frag_step 2 interleaves two sources fragment by
// fragment.  transpose: the source is read as [cols][rows].
struct TgPack {
	const void *src;
	int src_f32;             // source dtype: 0 bfloat16, 1 float32
	int src_ld;              // elements per source row
	int rows, cols;          // destination rows and columns written (padded sizes)
	int rsrc, ksrc;          // source rows / columns (bounds)
	int g, gp, kg, kgp;
	int frag_step, frag_off;
	int transpose;
	float add;               // added to every element that exists
};
void tg_launch_pack(const TgMat &dst, int dt, const TgPack &p, hipStream_t s);
// the same mapping into plain rows of floats: dst[i * ld + j] = source row and column of (i, j), 0 in the padding
void tg_launch_unpack_f32(float *dst, int ld, const TgPack &p, hipStream_t s);

// ---- one-row products of a decode step ---------------------------------------------------------------------------------
// y = W x for one vector, or for `nz` of them at once (head blocks, experts).  A workgroup owns one tile of 16 outputs (two
// for the gate|up pair) over its part of K, or, where there are thousands of tiles, four of them.  The vector is prepared by
// every workgroup in a prologue and held in LDS.
#define TG_VEC_MERGE_MAX 16        // attention partials a prologue merges
#define TG_VEC_MERGE_HEADS_MAX 64  // heads that TG_VP_MERGE_HEADS serves
enum {
	TG_VP_PLAIN = 0,   // x[z]
	TG_VP_DYT,         // residual sum, then the element-wise tanh norm
	TG_VP_RMS,         // residual sum (its addend normed first where there is a weight for it), then the root mean square norm
	TG_VP_HEADNORM,    // heads normalised by their root mean square, times silu(gate) or sigmoid(gate)
	TG_VP_MERGE,       // merged attention partials of head z
	TG_VP_MERGE_HEADS, // the same of all heads, side by side (vdimp elements each): groups of `group` heads, each padded to 16
	TG_VP_EXPERT       // x, for the z-th of the experts that the router's logits select
};
enum {
	TG_VE_STORE = 0,
	TG_VE_GELU,        // the exact gelu
	TG_VE_SWIGLU,      // silu(gate) * up of a tile pair
	TG_VE_LOGITS,      // store + maximum of the workgroup's outputs
	TG_VE_GATE,        // times sigmoid(gate[z])
	TG_VE_WEIGHTED     // expert sel[z], times wgt[z]
};
struct TgVec {
	const void *W;
	int kfrags, ntiles;        // fragments along K; tiles of 16 outputs (tile pairs: of the pair's 32 rows)
	int nz;
	long long zfrags;          // fragments between the matrices of consecutive z (or experts)
	int ksplit;                // parts of K; part p writes y + p * part_stride
	// inputs
	const float *x;
	int x_zstride;
	const float *pend;         // DYT: x + mult * (sum of nparts vectors, pend_stride apart) is the new residual
	int nparts, pend_stride;
	float mult;
	const float *nw, *nb;      // DYT: weight and bias; RMS, HEADNORM: nw = the norm's weight
	const float *post;         // RMS: weight of the norm of the sum of parts before it is added (mult is then unused)
	int width;                 // RMS: elements that the means are over (K without its padding)
	float alpha;
	float *x_out, *h_out;      // DYT, RMS: the new residual and the normalised vector (may be null)
	const void *embed;         // DYT, RMS: x is row ctr[4] of this table instead (null: x)
	int embed_ld, vocab;
	float embed_scale;         // RMS: factor of that row
	const int *ctr;
	const float *gate;         // HEADNORM: gate vector laid out like x; GATE: one value per z
	int gate_sigmoid;          // HEADNORM: sigmoid(gate) instead of silu(gate)
	int vdim, vdimp;           // HEADNORM: head size and its padded size
	float eps;
	const float *part_acc, *part_ml;  // MERGE: [nmerge][heads padded to 16][x_zstride], [nmerge][heads padded to 16][2]
	int nmerge, heads16, group, heads;  // MERGE_HEADS: heads per group, real heads; heads16 counts the padded heads of all groups
	const float *logits, *correction;  // EXPERT
	int experts, top;
	float rscale;
	int *sel;                  // EXPERT: written by one workgroup; WEIGHTED: read
	float *wgt;
	// output
	const float *bias;         // STORE: added to the outputs (null: none)
	float *y;
	int y_zstride, part_stride;
	int nout;                  // LOGITS: outputs that exist (the rest is padding)
	float *blk_val;
	int *blk_idx;
};
void tg_launch_vec(const TgVec &v, int dt, int pro, int epi, hipStream_t s);
int tg_vec_blocks(const TgVec &v, int epi);  // workgroups along x (the number of blk_val entries of TG_VE_LOGITS)
int tg_vec_ksplit(int ntiles, int nz, int kfrags, int n_cu);

// ---- tiled products ------------------------------------------------------------------------------------------------------
// C = A W^T, A [M][lda] row-major in the model's format.
enum {
	TG_GE_STORE = 0,   // columns below n_split to C (format), the rest to C2 (fp32)
	TG_GE_F32,         // C2 (fp32)
	TG_GE_RESID,       // C2 += mult * result
	TG_GE_SWIGLU,      // fragments alternate gate, up: C = silu(gate) * up
	TG_GE_GELU,        // C = the exact gelu of the result
	TG_GE_TRANS        // C^T: C[n][ldc], columns in the key order of the attention operand (tg_latent.h)
};
struct TgGemm {
	const void *A;
	int lda;               // elements
	const void *W;
	int M, K, N;           // padded K and N
	void *C;
	int ldc;
	float *C2;
	int ldc2, n_split;
	float mult;
	const float *bias;     // STORE: added to the columns below n_split (null: none)
	int rows_out;          // TRANS: output columns written (>= M: the last row repeats)
	// grouped: tile t of the list covers rows [tiles[t].y, tiles[t].z) with the matrix of group tiles[t].x
	const int4 *tiles;     // null: one matrix
	const int *ntiles;     // device: tiles in the list
	int max_tiles;
	int tile_rows;         // rows per tile: 128, 64 or 32
	const int *row_src;    // row r of the product reads row row_src[r] of A (null: r)
	long long group_frags; // fragments between the matrices of consecutive groups
};
void tg_launch_linear(const TgGemm &g, int dt, int epi, hipStream_t s);
