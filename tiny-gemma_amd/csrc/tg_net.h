// Layer-list models: decoder-only models described by a folder with config.json and model.safetensors, whose layers are
// named one by one.  tg_net.hip holds the registry of designs, the loader, the per-sequence state and the kernel sequences;
// tg_api.hip puts them behind tg_model and tg_session.  Nothing here is part of the C ABI.
#pragma once

#include <functional>

#include "tg_linear.h"

enum { TG_MIX_LATENT = 0, TG_MIX_GLA, TG_MIX_DELTA, TG_MIX_ATTN };
enum { TG_FF_NONE = 0, TG_FF_MOE, TG_FF_DENSE };
// TG_NORM_TANH: an element-wise tanh before each sublayer, whose output is added times residual_mult.
// TG_NORM_RMS: root mean square norms before and after each sublayer, weights stored around zero.
enum { TG_NORM_TANH = 0, TG_NORM_RMS };

struct TgMixerCfg {
	int kind = 0, heads = 0, dim = 0, vdim = 0;
	int rank = 0;         // latent: kv_rank; gla, delta: rank of the decay projection (from its tensor)
	float scale = 0.0f;   // latent, attention: factor of q . k
	float tau = 1.0f;     // gla
	int kv_heads = 0;     // delta: q/k heads; attention: key heads
	int q_rank = 0;       // latent: size of the query's latent (0: the query is a projection, and heads have gates)
	int rot_dim = 0;      // latent: size of the rotated part (0: no positions)
	int rot_dims = 0;     // rotated dimensions
	double rot_base = 0;
	int window = 1 << 30; // latent, attention: newest token and window - 1 before it
	int taps = 0;         // delta: convolution
	int gate_rank = 0;    // delta: rank of the output gate (from its tensor)
	int dimp() const { return tg_up(dim, 32); }
	int vdimp() const { return tg_up(vdim, 32); }
	int rotp() const { return tg_up(kind == TG_MIX_ATTN ? rot_dims : rot_dim, 32); }   // rotated part of a cache row
};
struct TgMoeCfg {
	int experts = 0, top = 0, ff = 0;  // (a dense feed-forward: ff only)
	float scale = 1.0f;
	int ffp() const { return tg_up(ff, 64); }
};
struct TgNetLayerCfg {
	TgMixerCfg mix;
	int mlp = TG_FF_NONE;
	TgMoeCfg moe;
	int weights_of = -1;
};
struct TgNetCfg {
	std::string arch;
	int width = 0, vocab = 0;
	int norm = TG_NORM_TANH;
	float eps = 0.0f, residual_mult = 1.0f, embed_scale = 1.0f;
	std::vector<TgNetLayerCfg> layers;
	std::vector<int> runs;  // the layer of every layer run, in order; each run has its own cache or state
	int wp() const { return tg_up(width, 64); }
};

// What the end of a forward leaves for the sampler: logits and their maxima per workgroup of the head, and the device
// counters ([0] position, [4] token) that a decode step reads.
struct TgHead {
	float *logits;
	float *blk_val;
	int *blk_idx;
	int *ctr;
};

struct TgNet;
struct TgNetSeq;
typedef std::function<int(void *dst, size_t off, size_t len)> TgFill;
// tg_api.hip: bytes to the device through the pinned staging buffers of the weight loader
int tg_stage_image(uint8_t *d_raw, size_t n, const TgFill &fill);

bool tg_net_known(const std::string &arch);
int tg_net_open(const char *dir, int dt, int n_cu, hipStream_t s, TgNet **out);
void tg_net_free(TgNet *n);
const TgNetCfg &tg_net_cfg(const TgNet *n);
int tg_net_dtype(const TgNet *n);
int tg_net_head_blocks(const TgNet *n);
int tg_net_vocab_padded(const TgNet *n);
// bytes of weights a decode step reads, and launches it takes (for the choice of its launch form)
void tg_net_step_cost(const TgNet *n, double *bytes, int *launches);

int tg_net_seq_create(TgNet *n, int capacity, TgNetSeq **out);
int tg_net_seq_reset(TgNetSeq *q);
void tg_net_seq_free(TgNetSeq *q);
void tg_net_seq_release_workspace(TgNetSeq *q);
// n tokens behind pos earlier ones.  want: positions among them whose logits go to `logits` (host, [n_want][vocab]).
// Leaves the last token's logits and maxima in h.  taps: keep the residual stream after every block.
int tg_net_rows(TgNetSeq *q, const int32_t *ids, int n, int pos, const int32_t *want, int n_want, float *logits, const TgHead &h, bool taps);
// one token, h.ctr[4], at position pos (pos_bound: positions the launch must serve; host_pos false: the kernels read h.ctr[0])
int tg_net_step(TgNetSeq *q, const TgHead &h, int pos, bool host_pos, int pos_bound);
// a captured step was replayed: the residual stream kept is that of a step again
void tg_net_replayed(TgNetSeq *q);
// residual stream after block b of the last forward (as tg_session_tap); rows must match what was kept
int tg_net_tap(TgNetSeq *q, int b, float *out, int rows);
