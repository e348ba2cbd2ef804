// Mixture of experts with sigmoid scores and a correction that only the choice sees (tg_moe.hip), and the row step around
// it: residual sums and the element-wise tanh norm of many rows.
#pragma once

#include "tg_linear.h"

#define TG_MOE_MAX_EXPERTS 1024
#define TG_MOE_BLOCK 16  // tokens per routing workgroup

// Routing of n tokens: logits [n][ld] fp32.  Expert e's rows are the slots [offset(e), offset(e + 1)); tiles of tile_rows slots
// of one expert each, as the grouped products take them.
struct TgMoeRoute {
	const float *logits;
	int ld;
	const float *correction;
	int n, experts, top, tile_rows;
	float scale;
	int *sel;       // [n][top] chosen experts
	float *wgt;     // [n][top] their weights
	int *slot;      // [n][top] where their rows are (first the index inside the block's share of the expert)
	int *row_src;   // [n * top] token of a slot
	int *count;     // [blocks][experts], then the block's first slot of the expert
	int4 *tiles;    // {expert, first slot, end slot, 0}
	int *ntiles;
};
int tg_moe_max_tiles(int n, int experts, int top, int tile_rows);
void tg_launch_moe_route(const TgMoeRoute &r, hipStream_t s);

// n rows of the fp32 residual x [.][ldx]: optionally x = table row of ids[t], optionally x += mult * (weighted sum of the
// token's expert rows), then out = tanh(alpha x) w + b in the model's format (out may be null).  gather: row t of out
// comes from row gather[t] of x (x is then left alone).  (Padding: zero in x, the norm and the table.)
struct TgRowsDyt {
	float *x;
	int ldx, n;
	const int *gather;
	const void *embed;
	const int *ids;
	int vocab;
	const void *y;        // [slots][ldx] expert outputs, null: none
	const int *slot;      // [n][top]
	const float *wgt;
	int top;
	float mult, alpha;
	const float *nw, *nb; // [ldx]
	void *out;            // [n][ldx]
};
void tg_launch_rows_dyt(const TgRowsDyt &r, int dt, hipStream_t s);
