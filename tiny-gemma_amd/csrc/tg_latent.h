// Latent attention (tg_latent.hip): the cache holds one normalised latent row c per token, keys and values of every head
// are linear in it (k = Wuk c, v = Wuv c), no positions.  Causal softmax over everything cached; a head's output is
// multiplied by the sigmoid of its gate.
//
// One token: the head's query is taken through Wuk once (q' = Wuk^T q), so that scores and value sums are taken on the
// latent rows themselves, shared by all heads; Wuv is applied to the merged sum.  Many tokens: keys and transposed values of
// the whole context are products of the cache, then tiled attention per head.
#pragma once

#include "tg_linear.h"

#define TG_LATENT_MAX_PARTS TG_VEC_MERGE_MAX  // partials that the value product merges in its prologue
#define TG_LATENT_MAX_BLOCKS 128   // key parts per launch
#define TG_LATENT_TILE 32
#define TG_LATENT_LDS_MAX (150 * 1024)
#define TG_LATENT_HEAD_MAX 256     // largest padded head size of the tiled kernel

struct TgLatentStep {
	int heads, rank, rankp;        // rankp: elements between cache rows (padded to 64)
	const float *q;                // [heads][rankp] q' (after the product with Wuk^T)
	const float *dkv;              // [rank] the new token's latent before its norm
	const float *norm;             // [rank]
	float eps, scale;
	void *cache;                   // [capacity][rankp] in the model's format; the new row is written here
	const int *ctr;                // device counters; ctr[0] = position
	int host_pos;                  // the position, or -1: read the counter
	int chunk, nb;                 // keys per part (multiple of TG_LATENT_TILE), parts
	float *part_acc, *part_ml;     // [nb][heads16][rankp], [nb][heads16][2]
};
void tg_launch_latent_step(const TgLatentStep &a, int dt, hipStream_t s);
size_t tg_latent_step_lds(int rankp, int dt);  // LDS the step asks for, besides its static 7 KiB
// folds nb > TG_LATENT_MAX_PARTS partials into one
void tg_launch_latent_fold(const float *acc, const float *ml, int nb, int heads16, int rankp, float *out_acc, float *out_ml, hipStream_t s);

// cache rows of n tokens from raw latents
void tg_launch_latent_rows(const float *dkv, int ld, int n, int rank, int rankp, const float *norm, float eps, int dt, void *cache_rows,
                           hipStream_t s);

// q [n][ldq], k [context][ldk]: heads side by side, dimp apart; vt [heads * vdimp][ldv]: the values transposed, keys of every block
// of 32 (bf16: order 8 * ((t % 16) / 4) + 4 * (t / 16) + t % 4) or 16 (fp32: as they are) in operand order, finite up to the
// next multiple of 64 keys; gate [n][ld_gate] fp32, one per head; query i sees keys 0 ... past + i; out [n][ldo], columns behind
// the heads are cleared.
struct TgLatentRows {
	const void *q, *k, *vt;
	int ldq, ldk, ldv;
	const float *gate;
	int ld_gate;
	void *out;
	int ldo;
	int n, past, heads, dimp, vdimp;
	float scale;
};
void tg_launch_latent_attention(const TgLatentRows &a, int dt, hipStream_t s);
