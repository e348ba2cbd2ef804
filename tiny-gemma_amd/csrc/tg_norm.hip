// Row norms and rotary tables: tg_norm.h.

#include "tg_norm.h"

namespace {

// Four columns per lane and pass, NP passes held in registers; a row is the work of WPR waves.
template <class TR, int WPR, int NP>
__global__ __launch_bounds__(256) void rows_rms_kernel(TgRowsRms r) {
	typedef typename TR::T T;
	__shared__ float s_red[2][4];
	const int w = threadIdx.x >> 6, t = blockIdx.x * (4 / WPR) + w / WPR, lane = threadIdx.x & (64 * WPR - 1);
	if (t >= r.n) return;  // (whole rows: with WPR = 4 the whole workgroup)
	auto total = [&](float v, int slot) {
		v = tg_wave_sum(v);
		if constexpr (WPR == 4) {
			if ((threadIdx.x & 63) == 0) s_red[slot][w] = v;
			__syncthreads();
			v = (s_red[slot][0] + s_red[slot][1]) + (s_red[slot][2] + s_red[slot][3]);
		}
		return v;
	};
	float *xr = r.x + (size_t)(r.gather ? r.gather[t] : t) * r.ldx;
	int id = 0;
	if (r.embed) {
		id = r.ids[t];
		id = id < 0 ? 0 : (id >= r.vocab ? r.vocab - 1 : id);
	}
	f32x4_t x[NP], y[NP];
#pragma unroll
	for (int i = 0; i < NP; i++) {
		const int c = 4 * (lane + i * 64 * WPR), cc = min(c, r.cols - 4);
		if (r.embed) {
			x[i] = tg_load4((const __bf16 *)r.embed + (size_t)id * r.ldx + cc);
#pragma unroll
			for (int e = 0; e < 4; e++) x[i][e] *= r.embed_scale;
		} else {
			x[i] = tg_load4(xr + cc);
		}
		if (c >= r.cols) x[i] = f32x4_t{0, 0, 0, 0};
		if (r.y) {
			y[i] = tg_load4(r.y + (size_t)t * r.ldy + min(c, r.cols - 4));
			if (c >= r.cols) y[i] = f32x4_t{0, 0, 0, 0};
		}
	}
	if (r.y) {
		float ss = 0.0f;
#pragma unroll
		for (int i = 0; i < NP; i++)
#pragma unroll
			for (int e = 0; e < 4; e++) ss = fmaf(y[i][e], y[i][e], ss);
		const float inv = 1.0f / sqrtf(total(ss, 0) / (float)r.width + r.eps);
#pragma unroll
		for (int i = 0; i < NP; i++) {
			const int c = 4 * (lane + i * 64 * WPR);
			const f32x4_t pw = tg_load4(r.post + min(c, r.cols - 4));
#pragma unroll
			for (int e = 0; e < 4; e++) x[i][e] += y[i][e] * inv * pw[e];
		}
	}
	if (r.embed || r.y) {
#pragma unroll
		for (int i = 0; i < NP; i++) {
			const int c = 4 * (lane + i * 64 * WPR);
			if (c < r.cols) tg_store4(xr + c, x[i]);
		}
	}
	if (!r.out) return;
	float ss = 0.0f;
#pragma unroll
	for (int i = 0; i < NP; i++)
#pragma unroll
		for (int e = 0; e < 4; e++) ss = fmaf(x[i][e], x[i][e], ss);
	const float inv = 1.0f / sqrtf(total(ss, 1) / (float)r.width + r.eps);
#pragma unroll
	for (int i = 0; i < NP; i++) {
		const int c = 4 * (lane + i * 64 * WPR);
		const f32x4_t nw = tg_load4(r.nw + min(c, r.cols - 4));
		f32x4_t h;
#pragma unroll
		for (int e = 0; e < 4; e++) h[e] = x[i][e] * inv * nw[e];
		if (c < r.cols) tg_store4((T *)r.out + (size_t)t * r.ldo + c, h);
	}
}

template <class TR>
void launch_rms(const TgRowsRms &r, hipStream_t s) {
	const int w = r.cols;
	const dim3 one((unsigned)((r.n + 3) / 4)), four((unsigned)r.n);
	if (w <= 256) hipLaunchKernelGGL((rows_rms_kernel<TR, 1, 1>), one, dim3(256), 0, s, r);
	else if (w <= 512) hipLaunchKernelGGL((rows_rms_kernel<TR, 1, 2>), one, dim3(256), 0, s, r);
	else if (w <= 1024 && r.n >= 2048) hipLaunchKernelGGL((rows_rms_kernel<TR, 1, 4>), one, dim3(256), 0, s, r);
	else if (w <= 1024) hipLaunchKernelGGL((rows_rms_kernel<TR, 4, 1>), four, dim3(256), 0, s, r);
	else if (w <= 2048) hipLaunchKernelGGL((rows_rms_kernel<TR, 4, 2>), four, dim3(256), 0, s, r);
	else if (w <= 4096) hipLaunchKernelGGL((rows_rms_kernel<TR, 4, 4>), four, dim3(256), 0, s, r);
	else hipLaunchKernelGGL((rows_rms_kernel<TR, 4, 8>), four, dim3(256), 0, s, r);
}

__global__ __launch_bounds__(256) void rot_table_kernel(float2 *table, int positions, int half, double log2_base) {
	const long long total = (long long)positions * half;
	for (long long e = (long long)blockIdx.x * 256 + threadIdx.x; e < total; e += (long long)gridDim.x * 256) {
		const int p = (int)(e / half), i = (int)(e - (long long)p * half);
		const double a = (double)p * exp2(-(double)i / (double)half * log2_base);
		table[e] = float2{(float)cos(a), (float)sin(a)};
	}
}

}  // namespace

void tg_launch_rows_rms(const TgRowsRms &rows, int dt, hipStream_t s) {
	TgRowsRms r = rows;
	if (!r.cols) r.cols = r.ldx;
	if (dt == TG_DT_BF16) launch_rms<TgB16>(r, s);
	else launch_rms<TgF32>(r, s);
}

void tg_launch_rot_table(float2 *table, int positions, int dims, double base, hipStream_t s) {
	const int half = dims / 2;
	const long long n = ((long long)positions * half + 255) / 256;
	hipLaunchKernelGGL(rot_table_kernel, dim3((unsigned)(n < 4096 ? n : 4096)), dim3(256), 0, s, table, positions, half, log2(base));
}
