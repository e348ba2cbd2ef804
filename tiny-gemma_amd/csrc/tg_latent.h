// Attention on shared rows (tg_latent.hip).  Per token the cache holds, for each of `groups` key/value heads, one row
// [value part | rotated key part], the parts padded; a query head scores q . value part + q' . rotated part and sums the value
// parts.  Three mechanisms are laid out like this:
//   * latent attention: one group; the value part is the normalised latent c, keys and values of every head are linear in it
//     (k = Wuk c, v = Wuv c), no rotated part;
//   * latent attention with positions: the rotated part is a key part shared by all heads;
//   * grouped-query attention whose values are its keys before rotation: the value part is the key of the group, the rotated
//     part its first rotated dimensions; the query's own first dimensions meet the rotated part only.
// Causal softmax over everything cached or over the last `window` tokens; a head's output may be multiplied by the sigmoid of
// its gate.
//
// One token: scores and value sums are taken on the rows themselves; the latent's query is taken through Wuk once
// (q' = Wuk^T q) and Wuv is applied to the merged sum.  Many tokens: keys and transposed values of the context (of the part
// that a window can reach) are made from the cache, as products or by a row kernel, then tiled attention per head.
#pragma once

#include "tg_linear.h"

#define TG_LATENT_MAX_PARTS TG_VEC_MERGE_MAX  // partials that the value product merges in its prologue
#define TG_LATENT_MAX_BLOCKS 128   // key parts per launch
#define TG_LATENT_TILE 32
#define TG_LATENT_LDS_MAX (150 * 1024)
#define TG_LATENT_HEAD_MAX 256     // largest padded head size of the tiled kernel, and rotated part of a row

// Rotary positions: dims / 2 pairs of a vector, (2i, 2i + 1) or (i, i + dims / 2); elements behind them pass unchanged.
struct TgRot {
	const float2 *table;           // [position][dims / 2] cos, sin
	int dims, half_layout;
};
#define TG_NO_WINDOW (1 << 30)

struct TgLatentStep {
	int groups, heads;             // heads: query heads of one group (heads of group g: g * heads ...)
	int rank, rankp;               // value part: size and padded size (32)
	int rot_size, rotp;            // rotated part: size and padded size (32; 0: none)
	const float *q;                // [head][q_stride], its first rank elements; the first q_zero of them count as zero
	int q_stride, q_zero;
	const float *qr;               // [head][qr_stride] rotated part of the query before its rotation
	int qr_stride;
	const float *kv;               // [group][kv_stride] the new token's value part (before its norm)
	int kv_stride;
	const float *kr;               // [group][kr_stride] its rotated part before rotation
	int kr_stride;
	TgRot rot;
	const float *norm;             // [rank], null: the value part as it is
	float eps, scale;
	int window;                    // the newest token and window - 1 before it
	void *cache;                   // [capacity][groups][rankp + rotp] in the model's format; the new row is written here
	const int *ctr;                // device counters; ctr[0] = position
	int host_pos;                  // the position, or -1: read the counter
	int chunk, nb;                 // keys per part (multiple of TG_LATENT_TILE), parts
	float *part_acc, *part_ml;     // [nb][groups * heads16][rankp], [nb][groups * heads16][2]; heads16: heads padded to 16
	int rowp() const { return rankp + rotp; }
};
void tg_launch_latent_step(const TgLatentStep &a, int dt, hipStream_t s);
size_t tg_latent_step_lds(int rowp, int dt);  // LDS the step asks for, besides its static 7 KiB
// folds nb partials into one (heads: of all groups, padded); out: instead of a partial the normalised sums of the real heads,
// [groups * heads][out_stride]
void tg_launch_latent_fold(const float *acc, const float *ml, int nb, int heads_padded, int rankp, float *out_acc, float *out_ml, hipStream_t s);
void tg_launch_latent_finish(const float *acc, const float *ml, int nb, int groups, int heads, int rankp, float *out, int out_stride, hipStream_t s);

// cache rows of n tokens behind `past` earlier ones, from projections: kv [n][ld] with the groups' value parts kv_stride apart,
// kr likewise; f32: the projections are fp32, else in the model's format
struct TgLatentCacheRows {
	const void *kv, *kr;
	int ld, f32, kv_stride, kr_stride;
	int n, past, groups, rank, rankp, rot_size, rotp;
	TgRot rot;
	const float *norm;
	float eps;
	void *cache;
};
void tg_launch_latent_rows(const TgLatentCacheRows &a, int dt, hipStream_t s);

// rotates `count` vectors per row in place: rows [n][ld] in the model's format, vector i at column first + i * stride
void tg_launch_rot_rows(void *rows, int ld, int n, int past, int first, int count, int stride, const TgRot &rot, int dt, hipStream_t s);

// keys and transposed values of a key-value cache: token lo + t of n; k [n][groups * dimp], rotated; vt as below
struct TgKeyValues {
	const void *cache;
	int lo, n, groups, dimp, rot_size, rotp;
	void *k, *vt;
	int ldv;
};
void tg_launch_key_values(const TgKeyValues &a, int dt, hipStream_t s);

// q [n][ldq], heads side by side, dimp + rotp apart; k [context][ldk]: key heads side by side, dimp apart; kr [context][ldkr]: the
// rotated part that all heads share (rotp 0: none); vt [key heads * vdimp][ldv]: the values transposed, keys of every block
// of 32 (bf16: order 8 * ((t % 16) / 4) + 4 * (t / 16) + t % 4) or 16 (fp32: as they are) in operand order, finite up to the
// next multiple of 64 keys; gate [n][ld_gate] fp32, one per head (null: none); query i sees keys past + i - window + 1 ... past
// + i; query head h uses key head h / group; out [n][ldo], columns behind the heads are cleared.
struct TgLatentRows {
	const void *q, *k, *kr, *vt;
	int ldq, ldk, ldkr, ldv;
	const float *gate;
	int ld_gate;
	void *out;
	int ldo;
	int n, past, heads, group, dimp, rotp, vdimp;
	int window;
	float scale;
};
void tg_launch_latent_attention(const TgLatentRows &a, int dt, hipStream_t s);
