// Routing of a prefill's tokens to experts, and the row step between the blocks: tg_moe.h.

#include "tg_moe.h"

namespace {

// a wave per token; the workgroup counts its tokens' choices per expert
__global__ __launch_bounds__(256) void moe_route_kernel(TgMoeRoute r) {
	extern __shared__ __align__(16) float sm[];
	const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, E = r.experts;
	int *s_cnt = (int *)sm;
	float *s_choice = sm + E + w * E, *s_val = sm + 5 * E + w * r.top;
	int *s_sel = (int *)(sm + 5 * E + 4 * r.top) + w * r.top;
	for (int e = tid; e < E; e += 256) s_cnt[e] = 0;
	__syncthreads();
	for (int i = w; i < TG_MOE_BLOCK; i += 4) {
		const int t = blockIdx.x * TG_MOE_BLOCK + i;
		if (t < r.n) {
			const float *lg = r.logits + (size_t)t * r.ld;
			for (int e = lane; e < E; e += 64) s_choice[e] = tg_sigmoid(lg[e]) + r.correction[e];
			__builtin_amdgcn_wave_barrier();
			asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
			for (int e = lane; e < E; e += 64) {
				const float c = s_choice[e];
				int rank = 0;
				for (int o = 0; o < E; o++) {
					const float co = s_choice[o];
					rank += (co > c || (co == c && o < e)) ? 1 : 0;
				}
				if (rank < r.top) {
					s_sel[rank] = e;
					s_val[rank] = tg_sigmoid(lg[e]);
				}
			}
			__builtin_amdgcn_wave_barrier();
			asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
			for (int k = lane; k < r.top; k += 64) {
				float sum = 0.0f;
				for (int o = 0; o < r.top; o++) sum += s_val[o];
				const size_t at = (size_t)t * r.top + k;
				r.sel[at] = s_sel[k];
				r.wgt[at] = s_val[k] / (sum + 1e-20f) * r.scale;
				r.slot[at] = atomicAdd(&s_cnt[s_sel[k]], 1);
			}
		}
	}
	__syncthreads();
	for (int e = tid; e < E; e += 256) r.count[(size_t)blockIdx.x * E + e] = s_cnt[e];
}

// One workgroup: first slot of every (block, expert), and the tile list.  A thread per expert and segment of the blocks
// (ep = experts rounded up to a power of two, TG_MOE_MAX_EXPERTS / ep segments).
__global__ __launch_bounds__(TG_MOE_MAX_EXPERTS) void moe_offsets_kernel(TgMoeRoute r, int blocks, int ep) {
	__shared__ int s_seg[TG_MOE_MAX_EXPERTS], s_n[TG_MOE_MAX_EXPERTS], s_t[TG_MOE_MAX_EXPERTS];
	const int E = r.experts, tid = threadIdx.x, e = tid & (ep - 1), seg = tid / ep, segs = TG_MOE_MAX_EXPERTS / ep;
	const int per = (blocks + segs - 1) / segs, b0 = min(seg * per, blocks), b1 = min(b0 + per, blocks);
	const int ec = min(e, E - 1);
	int own = 0;
	for (int b = b0; b < b1; b += 8) {
		int c[8];
#pragma unroll
		for (int i = 0; i < 8; i++) c[i] = r.count[(size_t)min(b + i, b1 - 1) * E + ec];
#pragma unroll
		for (int i = 0; i < 8; i++) own += (b + i < b1 && e < E) ? c[i] : 0;
	}
	s_seg[tid] = own;
	__syncthreads();
	for (int o = 1; o < segs; o <<= 1) {  // inclusive sums over the segments of an expert
		const int v = seg >= o ? s_seg[tid - o * ep] : 0;
		__syncthreads();
		s_seg[tid] += v;
		__syncthreads();
	}
	const int cnt = s_seg[(segs - 1) * ep + e], nt = (cnt + r.tile_rows - 1) / r.tile_rows, before = s_seg[tid] - own;
	if (tid < ep) {
		s_n[e] = cnt;
		s_t[e] = nt;
	}
	__syncthreads();
	for (int o = 1; o < ep; o <<= 1) {  // inclusive sums over the experts
		const int a = tid < ep && e >= o ? s_n[e - o] : 0, b = tid < ep && e >= o ? s_t[e - o] : 0;
		__syncthreads();
		if (tid < ep) {
			s_n[e] += a;
			s_t[e] += b;
		}
		__syncthreads();
	}
	const int first = s_n[e] - cnt, t0 = s_t[e] - nt;
	if (e < E) {
		int run = first + before;
		for (int b = b0; b < b1; b++) {
			const int c = r.count[(size_t)b * E + e];
			r.count[(size_t)b * E + e] = run;
			run += c;
		}
		for (int i = seg; i < nt; i += segs) r.tiles[t0 + i] = int4{e, first + i * r.tile_rows, min(first + (i + 1) * r.tile_rows, first + cnt), 0};
	}
	if (tid == E - 1) *r.ntiles = s_t[e];
}

__global__ __launch_bounds__(256) void moe_scatter_kernel(TgMoeRoute r) {
	const int i = blockIdx.x * 256 + threadIdx.x;
	if (i >= r.n * r.top) return;
	const int t = i / r.top;
	const int slot = r.count[(size_t)(t / TG_MOE_BLOCK) * r.experts + r.sel[i]] + r.slot[i];
	r.slot[i] = slot;
	r.row_src[slot] = t;
}

// four columns per lane and pass; a wave per row, or where there are few rows (WPR = 4) a workgroup per row
template <class TR, int WPR>
__global__ __launch_bounds__(256) void rows_dyt_kernel(TgRowsDyt r) {
	typedef typename TR::T T;
	const int t = blockIdx.x * (4 / WPR) + (threadIdx.x >> 6) / WPR, lane = threadIdx.x & (64 * WPR - 1);
	if (t >= r.n) return;
	float *xr = r.x + (size_t)(r.gather ? r.gather[t] : t) * r.ldx;
	int id = 0;
	if (r.embed) {
		id = r.ids[t];
		id = id < 0 ? 0 : (id >= r.vocab ? r.vocab - 1 : id);
	}
	for (int c = 4 * lane; c < r.ldx; c += 256 * WPR) {
		f32x4_t x = r.embed ? tg_load4((const __bf16 *)r.embed + (size_t)id * r.ldx + c) : tg_load4(xr + c);
		if (r.y) {
			f32x4_t add = {0, 0, 0, 0};
			for (int k0 = 0; k0 < r.top; k0 += 8) {
				f32x4_t y[8];
				float g[8];
#pragma unroll
				for (int k = 0; k < 8; k++) {
					const size_t at = (size_t)t * r.top + min(k0 + k, r.top - 1);
					g[k] = k0 + k < r.top ? r.wgt[at] : 0.0f;
					y[k] = tg_load4((const T *)r.y + (size_t)r.slot[at] * r.ldx + c);
				}
#pragma unroll
				for (int k = 0; k < 8; k++)
#pragma unroll
					for (int e = 0; e < 4; e++) add[e] = fmaf(g[k], y[k][e], add[e]);
			}
#pragma unroll
			for (int e = 0; e < 4; e++) x[e] = x[e] + r.mult * add[e];
		}
		if (r.embed || r.y) tg_store4(xr + c, x);
		if (r.out) {
			const f32x4_t nw = tg_load4(r.nw + c), nb = tg_load4(r.nb + c);
			f32x4_t h;
#pragma unroll
			for (int e = 0; e < 4; e++) h[e] = tanhf(r.alpha * x[e]) * nw[e] + nb[e];
			tg_store4((T *)r.out + (size_t)t * r.ldx + c, h);
		}
	}
}

}  // namespace

int tg_moe_max_tiles(int n, int experts, int top, int tile_rows) {
	const int rows = n * top;
	return rows / tile_rows + (experts < rows ? experts : rows);
}

void tg_launch_moe_route(const TgMoeRoute &r, hipStream_t s) {
	const int blocks = (r.n + TG_MOE_BLOCK - 1) / TG_MOE_BLOCK;
	const size_t lds = sizeof(float) * (5 * (size_t)r.experts + 8 * (size_t)r.top);
	hipLaunchKernelGGL(moe_route_kernel, dim3((unsigned)blocks), dim3(256), lds, s, r);
	int ep = 1;
	while (ep < r.experts) ep *= 2;
	hipLaunchKernelGGL(moe_offsets_kernel, dim3(1), dim3(TG_MOE_MAX_EXPERTS), 0, s, r, blocks, ep);
	hipLaunchKernelGGL(moe_scatter_kernel, dim3((unsigned)((r.n * r.top + 255) / 256)), dim3(256), 0, s, r);
}

void tg_launch_rows_dyt(const TgRowsDyt &r, int dt, hipStream_t s) {
	const bool few = r.n < 2048;
	const dim3 grid((unsigned)(few ? r.n : (r.n + 3) / 4));
	if (dt == TG_DT_BF16) {
		if (few) hipLaunchKernelGGL((rows_dyt_kernel<TgB16, 4>), grid, dim3(256), 0, s, r);
		else hipLaunchKernelGGL((rows_dyt_kernel<TgB16, 1>), grid, dim3(256), 0, s, r);
	} else {
		if (few) hipLaunchKernelGGL((rows_dyt_kernel<TgF32, 4>), grid, dim3(256), 0, s, r);
		else hipLaunchKernelGGL((rows_dyt_kernel<TgF32, 1>), grid, dim3(256), 0, s, r);
	}
}
