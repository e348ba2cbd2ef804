// Root mean square norms of many rows, with the residual sums around them, and the tables of rotary positions
// (tg_norm.hip).
#pragma once

#include "tg_linear.h"

#define TG_RMS_WIDTH_MAX 7168  // longest vector a one-row product norms in its prologue (bounded by its LDS)

// n rows of the fp32 residual x [.][ldx]: optionally x = scale * table row of ids[t], optionally x += post-norm(y) (y fp32
// [n][ldy], normed with weight `post`), then out = norm(x) in the model's format (out may be null).  Weights are factors (a
// weight stored around zero has its one added at load).  gather: row t of out comes from row gather[t] of x, which is then left
// alone.  The padding between `width` and `cols` (0: ldx) columns is zero in x, y, the weights and the table.
struct TgRowsRms {
	float *x;
	int ldx, n, width, cols;
	const int *gather;
	const void *embed;     // bfloat16, [vocab][ldx]
	const int *ids;
	int vocab;
	float embed_scale;
	const float *y;
	int ldy;
	const float *post;
	const float *nw;
	float eps;
	void *out;             // [n][ldo], `cols` columns written
	int ldo;
};
void tg_launch_rows_rms(const TgRowsRms &r, int dt, hipStream_t s);

// table[p][i] = {cos, sin}(p * base^(-2 i / dims)), p < positions, i < dims / 2
void tg_launch_rot_table(float2 *table, int positions, int dims, double base, hipStream_t s);
