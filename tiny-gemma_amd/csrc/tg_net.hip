// Layer-list models: registry, loader, sequence state and kernel sequences (tg_net.h).

#include "tg_net.h"

#include <fcntl.h>
#include <math.h>
#include <stdio.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <algorithm>
#include <map>

#include "tg_gla.h"
#include "tg_json.h"
#include "tg_latent.h"
#include "tg_moe.h"
#include "tg_norm.h"

namespace {

constexpr int SLICE = 4096;         // tokens per pass of a long portion (bounds the workspace)
constexpr int WANT_ROWS = 256;      // logits rows per product
constexpr int TAP_MAX_ROWS = 1024;  // longest portion whose residual stream is kept

// ---- configuration ---------------------------------------------------------------------------------------------------------
int bad(const std::string &what) { return tg_fail(TG_ERR_BAD_ARG, what); }

const TgJson *member(const TgJson *o, const char *key) { return o && o->is_object() ? o->get(key) : nullptr; }

int need_number(const TgJson *o, const char *key, const std::string &where, double *out) {
	const TgJson *v = member(o, key);
	if (!v || v->kind != TgJson::Number) return bad("config.json: " + where + " needs the number '" + key + "'");
	*out = v->num;
	return TG_OK;
}
int need_size(const TgJson *o, const char *key, const std::string &where, int *out) {
	double d = 0;
	if (int rc = need_number(o, key, where, &d)) return rc;
	if (!(d >= 1 && d <= 1 << 24) || d != floor(d)) return bad("config.json: '" + std::string(key) + "' of " + where + " is not a size");
	*out = (int)d;
	return TG_OK;
}
int need_float(const TgJson *o, const char *key, const std::string &where, float *out) {
	double d = 0;
	if (int rc = need_number(o, key, where, &d)) return rc;
	*out = (float)d;
	return TG_OK;
}

// Madevik: gated linear attention and latent attention layers in any order, element-wise tanh norms, mixtures of experts
// with sigmoid scores, layers that share another layer's weights.
int parse_madevik(const TgJson &j, TgNetCfg *c) {
	if (int rc = need_size(&j, "width", "the model", &c->width)) return rc;
	if (int rc = need_size(&j, "vocab", "the model", &c->vocab)) return rc;
	if (int rc = need_float(&j, "residual_mult", "the model", &c->residual_mult)) return rc;
	if (int rc = need_float(member(&j, "norm"), "eps", "'norm'", &c->eps)) return rc;
	const TgJson *ls = member(&j, "layers");
	if (!ls || ls->kind != TgJson::Array || ls->items.empty()) return bad("config.json: no 'layers'");
	for (size_t i = 0; i < ls->items.size(); i++) {
		const TgJson &l = ls->items[i];
		const std::string where = "layer " + std::to_string(i);
		TgNetLayerCfg lc;
		const TgJson *type = member(&l, "type"), *mix = member(&l, "mixer"), *mlp = member(&l, "mlp"), *of = member(&l, "weights_of");
		if (!type || type->kind != TgJson::String) return bad("config.json: " + where + " has no 'type'");
		if (int rc = need_size(mix, "heads", where, &lc.mix.heads)) return rc;
		if (int rc = need_size(mix, "dim", where, &lc.mix.dim)) return rc;
		if (int rc = need_size(mix, "vdim", where, &lc.mix.vdim)) return rc;
		if (type->str == "latent_attention") {
			lc.mix.kind = TG_MIX_LATENT;
			if (int rc = need_size(mix, "kv_rank", where, &lc.mix.rank)) return rc;
			if (int rc = need_float(mix, "scale", where, &lc.mix.scale)) return rc;
			if (lc.mix.dimp() > TG_LATENT_HEAD_MAX || lc.mix.vdimp() > TG_LATENT_HEAD_MAX)
				return tg_fail(TG_ERR_UNSUPPORTED_SHAPE, where + ": latent attention heads above " + std::to_string(TG_LATENT_HEAD_MAX));
		} else if (type->str == "gla") {
			lc.mix.kind = TG_MIX_GLA;
			if (int rc = need_float(mix, "tau", where, &lc.mix.tau)) return rc;
			if (lc.mix.vdimp() > TG_GLA_VDIM_MAX) return tg_fail(TG_ERR_UNSUPPORTED_SHAPE, where + ": value size above " + std::to_string(TG_GLA_VDIM_MAX));
		} else {
			return tg_fail(TG_ERR_UNSUPPORTED_SHAPE, where + ": unknown mixer '" + type->str + "'");
		}
		if (mlp && !mlp->is_null()) {
			const TgJson *kind = member(mlp, "kind"), *r = member(mlp, "router");
			if (!kind || kind->str != "moe") return tg_fail(TG_ERR_UNSUPPORTED_SHAPE, where + ": unknown feed-forward");
			lc.mlp = TG_FF_MOE;
			if (int rc = need_size(member(mlp, "expert"), "ff", where, &lc.moe.ff)) return rc;
			if (int rc = need_size(r, "experts", where, &lc.moe.experts)) return rc;
			if (int rc = need_size(r, "top", where, &lc.moe.top)) return rc;
			if (int rc = need_float(r, "scale", where, &lc.moe.scale)) return rc;
			if (lc.moe.top > lc.moe.experts) return bad("config.json: " + where + " chooses more experts than it has");
			if (lc.moe.experts > TG_MOE_MAX_EXPERTS) return tg_fail(TG_ERR_UNSUPPORTED_SHAPE, where + ": too many experts");
		}
		if (of && of->kind == TgJson::Number) {
			lc.weights_of = (int)of->num;
			if (lc.weights_of < 0 || lc.weights_of >= (int)ls->items.size() || lc.weights_of == (int)i)
				return bad("config.json: " + where + " shares the weights of no other layer");
		}
		c->layers.push_back(lc);
	}
	for (size_t i = 0; i < c->layers.size(); i++) {
		// a chain of references ends at the layer that has tensors; the sharer must have its sizes
		int of = c->layers[i].weights_of;
		if (of < 0) continue;
		for (size_t k = 0; k < c->layers.size() && c->layers[(size_t)of].weights_of >= 0; k++) of = c->layers[(size_t)of].weights_of;
		if (c->layers[(size_t)of].weights_of >= 0) return bad("config.json: 'weights_of' goes round in a circle");
		const TgNetLayerCfg &a = c->layers[i], &b = c->layers[(size_t)of];
		if (a.mix.kind != b.mix.kind || a.mix.heads != b.mix.heads || a.mix.dim != b.mix.dim || a.mix.vdim != b.mix.vdim || a.mix.rank != b.mix.rank ||
		    a.mlp != b.mlp || a.moe.experts != b.moe.experts || a.moe.ff != b.moe.ff)
			return bad("config.json: layer " + std::to_string(i) + " differs from the layer whose weights it uses");
		c->layers[i].weights_of = of;
	}
	for (size_t i = 0; i < c->layers.size(); i++) c->runs.push_back((int)i);
	return TG_OK;
}

// Positions and window of an attention layer.  size: of the vector whose first dimensions are rotated.
int parse_rot_mask(const TgJson *mix, const std::string &where, int size, TgMixerCfg *m) {
	const TgJson *rot = member(mix, "rot"), *mask = member(mix, "mask");
	double base = 0;
	if (int rc = need_size(rot, "dims", where + ", 'rot'", &m->rot_dims)) return rc;
	if (int rc = need_number(rot, "base", where + ", 'rot'", &base)) return rc;
	m->rot_base = base;
	if (m->rot_dims % 2 != 0 || m->rot_dims > size || !(base > 0)) return bad("config.json: " + where + " has a bad 'rot'");
	if (mask && !mask->is_null())
		if (int rc = need_size(mask, "size", where + ", 'mask'", &m->window)) return rc;
	return need_float(mix, "scale", where, &m->scale);
}

// Tutelix: rotated latent attention with a latent query, grouped-query attention whose values are its keys, both in a window,
// and the gated delta rule, in any order; norms around each sublayer; dense feed-forwards; a run of layers that is passed several
// times.
int parse_tutelix(const TgJson &j, TgNetCfg *c) {
	c->norm = TG_NORM_RMS;
	if (int rc = need_size(&j, "width", "the model", &c->width)) return rc;
	if (int rc = need_size(&j, "vocab", "the model", &c->vocab)) return rc;
	if (int rc = need_float(member(&j, "embedding"), "scale", "'embedding'", &c->embed_scale)) return rc;
	if (int rc = need_float(member(&j, "norm"), "eps", "'norm'", &c->eps)) return rc;
	if (c->wp() > TG_RMS_WIDTH_MAX) return tg_fail(TG_ERR_UNSUPPORTED_SHAPE, "width above " + std::to_string(TG_RMS_WIDTH_MAX));
	const TgJson *ls = member(&j, "layers");
	if (!ls || ls->kind != TgJson::Array || ls->items.empty()) return bad("config.json: no 'layers'");
	for (size_t i = 0; i < ls->items.size(); i++) {
		const TgJson &l = ls->items[i];
		const std::string where = "layer " + std::to_string(i);
		TgNetLayerCfg lc;
		TgMixerCfg &m = lc.mix;
		const TgJson *type = member(&l, "type"), *mix = member(&l, "mixer"), *mlp = member(&l, "mlp");
		if (!type || type->kind != TgJson::String) return bad("config.json: " + where + " has no 'type'");
		if (int rc = need_size(mix, "heads", where, &m.heads)) return rc;
		if (int rc = need_size(mix, "dim", where, &m.dim)) return rc;
		if (int rc = need_size(mix, "vdim", where, &m.vdim)) return rc;
		if (type->str == "latent_attention") {
			m.kind = TG_MIX_LATENT;
			if (int rc = need_size(mix, "kv_rank", where, &m.rank)) return rc;
			if (int rc = need_size(mix, "q_rank", where, &m.q_rank)) return rc;
			if (int rc = need_size(mix, "rot_dim", where, &m.rot_dim)) return rc;
			if (int rc = parse_rot_mask(mix, where, m.rot_dim, &m)) return rc;
			if (m.dimp() + m.rotp() > TG_LATENT_HEAD_MAX || m.vdimp() > TG_LATENT_HEAD_MAX)
				return tg_fail(TG_ERR_UNSUPPORTED_SHAPE, where + ": latent attention heads above " + std::to_string(TG_LATENT_HEAD_MAX));
			if (tg_up(m.q_rank, 64) > TG_RMS_WIDTH_MAX)
				return tg_fail(TG_ERR_UNSUPPORTED_SHAPE, where + ": q_rank above " + std::to_string(TG_RMS_WIDTH_MAX));
		} else if (type->str == "attention") {
			m.kind = TG_MIX_ATTN;
			if (int rc = need_size(mix, "kv_heads", where, &m.kv_heads)) return rc;
			if (int rc = parse_rot_mask(mix, where, m.dim, &m)) return rc;
			if (m.vdim != m.dim) return bad("config.json: " + where + ": the values are the keys, 'vdim' must be 'dim'");
			if (m.dimp() > TG_LATENT_HEAD_MAX)
				return tg_fail(TG_ERR_UNSUPPORTED_SHAPE, where + ": attention heads above " + std::to_string(TG_LATENT_HEAD_MAX));
		} else if (type->str == "channel_delta") {
			m.kind = TG_MIX_DELTA;
			if (int rc = need_size(mix, "kv_heads", where, &m.kv_heads)) return rc;
			if (int rc = need_size(mix, "conv", where, &m.taps)) return rc;
			if (m.dimp() > TG_DELTA_DIM_MAX || m.vdimp() > TG_GLA_VDIM_MAX)
				return tg_fail(TG_ERR_UNSUPPORTED_SHAPE, where + ": key size above " + std::to_string(TG_DELTA_DIM_MAX) + " or value size above " +
				                                             std::to_string(TG_GLA_VDIM_MAX));
		} else {
			return tg_fail(TG_ERR_UNSUPPORTED_SHAPE, where + ": unknown mixer '" + type->str + "'");
		}
		if (m.kv_heads && m.heads % m.kv_heads != 0) return bad("config.json: " + where + ": 'heads' is no multiple of 'kv_heads'");
		if (mlp && !mlp->is_null()) {
			const TgJson *kind = member(mlp, "kind");
			if (!kind || kind->str != "dense") return tg_fail(TG_ERR_UNSUPPORTED_SHAPE, where + ": unknown feed-forward");
			lc.mlp = TG_FF_DENSE;
			if (int rc = need_size(mlp, "ff", where, &lc.moe.ff)) return rc;
		}
		c->layers.push_back(lc);
	}
	const int n = (int)c->layers.size();
	int start = 0, stop = 0, times = 1;
	const TgJson *loop = member(&j, "loop");
	if (loop && !loop->is_null()) {
		double a = 0;
		if (int rc = need_number(loop, "start", "'loop'", &a)) return rc;
		if (int rc = need_size(loop, "stop", "'loop'", &stop)) return rc;
		if (int rc = need_size(loop, "times", "'loop'", &times)) return rc;
		if (!(a >= 0 && a < stop) || a != floor(a) || stop > n || times > 4096) return bad("config.json: 'loop' is no run of layers");
		start = (int)a;
	}
	for (int i = 0; i < start; i++) c->runs.push_back(i);
	for (int t = 0; t < times; t++)
		for (int i = start; i < stop; i++) c->runs.push_back(i);
	for (int i = stop; i < n; i++) c->runs.push_back(i);
	return TG_OK;
}

// The designs this library knows, by config.json's "architecture".
struct Arch {
	const char *name;
	int (*parse)(const TgJson &, TgNetCfg *);
};
const Arch ARCHS[] = {{"Madevik", parse_madevik}, {"Tutelix", parse_tutelix}};

// ---- weights ---------------------------------------------------------------------------------------------------------------
struct Norm {
	float *w = nullptr, *b = nullptr;
	float alpha = 0.0f;
};
struct LayerW {
	Norm n1, n2, n1b, n2b;
	// gla: q | k | v | g | a1; latent: q | dkv | g, with a latent query dq | dkv | rotated key part; delta: q | k | v | g1 | b | a1;
	// attention: q | k
	TgMat in;
	float *in_b = nullptr;      // attention: bias
	int n_split = 0;            // rows of `in` whose prefill output is in the model's format; the rest is fp32
	TgMat out;
	float *hnorm = nullptr;     // gla: head norm; latent: norm of the latent
	float *a2 = nullptr, *a2b = nullptr;
	TgMat uk_t, uk, uv;         // latent: per head Wuk^T (blocks), Wuk, Wuv
	TgMat uq;                   // latent with a latent query
	float *qnorm = nullptr;
	TgMat g2;                   // delta: second half of the output gate, packed (rows) and plain, transposed (step)
	float *g2t = nullptr, *conv = nullptr, *a_log = nullptr;
	TgMat router, gate_up, down;  // dense: gate_up is up
	float *correction = nullptr;
};

int row_k_off(const TgMixerCfg &m) { return m.heads * m.dimp(); }
int row_v_off(const TgMixerCfg &m) { return 2 * m.heads * m.dimp(); }
int row_g_off(const TgMixerCfg &m) { return 2 * m.heads * m.dimp() + m.heads * m.vdimp(); }
int delta_channels(const TgMixerCfg &m) { return 2 * m.kv_heads * m.dimp() + m.heads * m.vdimp(); }
int value_width(const TgMixerCfg &m) { return m.heads * m.vdimp(); }
// the first position that a token at `pos` sees
int window_start(const TgMixerCfg &m, int pos) { return std::max(0, pos - m.window + 1); }

}  // namespace

struct TgNet {
	TgNetCfg cfg;
	int dt = 0, n_cu = 256;
	hipStream_t stream = nullptr;
	std::vector<LayerW> w;      // per layer; empty for layers that use another's
	std::vector<void *> owned;
	void *embed = nullptr;      // [vocab][wp] bfloat16
	Norm fin;
	TgMat head;
	const LayerW &lw(int l) const { return w[(size_t)(cfg.layers[(size_t)l].weights_of >= 0 ? cfg.layers[(size_t)l].weights_of : l)]; }
};

struct TgNetSeq {
	TgNet *net = nullptr;
	int capacity = 0;
	// per layer run: cache rows (tg_latent.h) [capacity][groups][value part | rotated part], or fp32 state [heads][dimp][vdimp], with
	// the convolution's last inputs [taps][channels] behind it (gated delta rule)
	std::vector<void *> state;
	std::vector<size_t> state_bytes;
	std::vector<TgRot> rot;     // per layer run
	std::vector<void *> tables; // rotary tables, one per (dims, base)
	void *ws = nullptr;         // decode buffers, one allocation
	float *xr = nullptr;        // [2R + 1][wp], R layer runs
	float *yin = nullptr, *pend_a = nullptr, *pend_b = nullptr, *hx = nullptr, *mix = nullptr, *qp = nullptr, *logits = nullptr, *u = nullptr,
	      *wgt = nullptr, *acc = nullptr, *ml = nullptr, *facc = nullptr, *fml = nullptr, *gate = nullptr, *qq = nullptr;
	int *sel = nullptr;
	void *pf = nullptr;         // prefill workspace, grown on demand
	size_t pf_bytes = 0;
	float *taps = nullptr;      // [2R + 1][rows][wp] of the last portion
	int tap_rows = 0;
};

namespace {

// ---- loader ----------------------------------------------------------------------------------------------------------------
struct Tensor {
	int f32 = 0;  // 0 bfloat16, 1 float32, 2 int32
	std::vector<long long> shape;
	size_t off = 0, bytes = 0;
};

struct Loader {
	TgNet *n;
	std::map<std::string, Tensor> t;
	const uint8_t *host = nullptr;  // the file's data section, mapped
	uint8_t *dev = nullptr;         // its copy on the device
	int rc = TG_OK;

	// the tensor, with its shape checked; a dimension of 0 in `shape` is read from the file
	const Tensor *get(const std::string &name, std::vector<int *> dims) {
		if (rc) return nullptr;
		auto it = t.find(name);
		if (it == t.end()) {
			rc = tg_fail(TG_ERR_BAD_ARG, "model.safetensors has no tensor '" + name + "'");
			return nullptr;
		}
		bool ok = it->second.shape.size() == dims.size();
		for (size_t i = 0; ok && i < dims.size(); i++) {
			if (*dims[i] == 0) *dims[i] = (int)it->second.shape[i];
			ok = it->second.shape[i] == *dims[i] && *dims[i] > 0;
		}
		if (!ok || it->second.f32 > 1) {
			rc = tg_fail(TG_ERR_BAD_ARG, "model.safetensors: tensor '" + name + "' has another shape or type than config.json asks for");
			return nullptr;
		}
		return &it->second;
	}
	const Tensor *get2(const std::string &name, int rows, int cols) { return get(name, {&rows, &cols}); }

	void *alloc(size_t bytes) {
		void *p = nullptr;
		if (!rc && hipMalloc(&p, bytes) != hipSuccess) rc = tg_fail(TG_ERR_HIP, "hipMalloc of a weight failed");
		if (p) n->owned.push_back(p);
		return p;
	}
	TgMat mat(int rows, int k) {
		TgMat m;
		m.n = rows;
		m.k = k;
		m.w = alloc((size_t)rows * k * tg_dt_bytes(n->dt));
		return m;
	}
	static TgPack pack_of(const void *src, int f32, int ld, int rsrc, int ksrc) {
		TgPack p;
		memset(&p, 0, sizeof(p));
		p.src = src;
		p.src_f32 = f32;
		p.src_ld = ld;
		p.rsrc = rsrc;
		p.ksrc = ksrc;
		p.frag_step = 1;
		return p;
	}
	// rows [row0, row0 + rows) of m from the tensor [r][c]; groups: see TgPack (0: one group)
	void put(const TgMat &m, int row0, int rows, const std::string &name, int r, int c, int g = 0, int gp = 0, int kg = 0, int kgp = 0,
	         int frag_step = 1, int frag_off = -1) {
		const Tensor *s = get2(name, r, c);
		if (!s) return;
		TgPack p = pack_of(dev + s->off, s->f32, c, r, c);
		p.rows = rows;
		p.cols = m.k;
		p.g = g ? g : r;
		p.gp = gp ? gp : rows;
		p.kg = kg ? kg : c;
		p.kgp = kgp ? kgp : m.k;
		p.frag_step = frag_step;
		p.frag_off = frag_off >= 0 ? frag_off : row0 / 16;
		tg_launch_pack(m, n->dt, p, n->stream);
	}
	// rows [row0, row0 + rows) of m from the n rows behind src0 of the tensor [r][c]
	void put_part(const TgMat &m, int row0, int rows, const std::string &name, int r, int c, int src0, int n) {
		const Tensor *s = get2(name, r, c);
		if (!s) return;
		TgPack p = pack_of(dev + s->off + (size_t)src0 * c * (s->f32 ? 4 : 2), s->f32, c, n, c);
		p.rows = rows;
		p.cols = m.k;
		p.g = n;
		p.gp = rows;
		p.kg = c;
		p.kgp = m.k;
		p.frag_off = row0 / 16;
		tg_launch_pack(m, this->n->dt, p, this->n->stream);
	}
	// d[j][i] = the tensor [r][c]'s element (i, j): c rows of ld floats, the tensor's rows in groups of g padded to gp
	void put_transposed(float *d, int ld, int cols, const std::string &name, int r, int c, int g, int gp) {
		const Tensor *s = get2(name, r, c);
		if (!s) return;
		TgPack p = pack_of(dev + s->off, s->f32, c, c, r);
		p.rows = p.g = p.gp = c;
		p.cols = cols;
		p.kg = g;
		p.kgp = gp;
		p.transpose = 1;
		tg_launch_unpack_f32(d, ld, p, n->stream);
	}
	// vector of `len` floats from [c], groups of kg padded to kgp; into d, or a new one
	float *vec(const std::string &name, int c, int len, int kg = 0, int kgp = 0, float add = 0.0f, float *d = nullptr) {
		const Tensor *s = get(name, {&c});
		if (!d) d = (float *)alloc((size_t)len * sizeof(float));
		if (rc) return nullptr;
		TgPack p = pack_of(dev + s->off, s->f32, c, 1, c);
		p.rows = 1;
		p.cols = len;
		p.g = p.gp = 1;
		p.kg = kg ? kg : c;
		p.kgp = kgp ? kgp : len;
		p.add = add;
		tg_launch_unpack_f32(d, len, p, n->stream);
		return d;
	}
	float scalar(const std::string &name) {
		auto it = t.find(name);
		if (rc) return 0.0f;
		if (it == t.end() || it->second.f32 > 1 || it->second.bytes != (it->second.f32 ? 4u : 2u)) {
			rc = tg_fail(TG_ERR_BAD_ARG, "model.safetensors has no scalar '" + name + "'");
			return 0.0f;
		}
		uint32_t u = 0;
		if (it->second.f32) memcpy(&u, host + it->second.off, 4);
		else {
			uint16_t h;
			memcpy(&h, host + it->second.off, 2);
			u = (uint32_t)h << 16;
		}
		float f;
		memcpy(&f, &u, 4);
		return f;
	}
	Norm norm(const std::string &name) {
		Norm r;
		if (n->cfg.norm == TG_NORM_RMS) {
			r.w = vec(name, n->cfg.width, n->cfg.wp(), 0, 0, 1.0f);
			return r;
		}
		r.w = vec(name, n->cfg.width, n->cfg.wp());
		r.b = vec(name + ".b", n->cfg.width, n->cfg.wp());
		r.alpha = scalar(name + ".alpha");
		return r;
	}

	void layer(int l) {
		TgNetLayerCfg &lc = n->cfg.layers[(size_t)l];
		TgMixerCfg &m = lc.mix;
		LayerW &w = n->w[(size_t)l];
		const std::string p = "l" + std::to_string(l) + ".", mp = p + "mix.";
		const int D = n->cfg.width, Dp = n->cfg.wp(), H = m.heads, dim = m.dim, dp = m.dimp(), vdim = m.vdim, vp = m.vdimp();
		const int ko = tg_up(H * vp, 64);
		w.n1 = norm(p + "norm1");
		if (m.kind == TG_MIX_GLA) {
			int d = D;
			m.rank = 0;
			get(mp + "a1", {&m.rank, &d});
			if (rc) return;
			const int r16 = tg_up(m.rank, 16), rank = m.rank;
			w.n_split = row_g_off(m) + H * vp;
			w.in = mat(w.n_split + r16, Dp);
			put(w.in, 0, H * dp, mp + "q", H * dim, D, dim, dp);
			put(w.in, row_k_off(m), H * dp, mp + "k", H * dim, D, dim, dp);
			put(w.in, row_v_off(m), H * vp, mp + "v", H * vdim, D, vdim, vp);
			put(w.in, row_g_off(m), H * vp, mp + "g", H * vdim, D, vdim, vp);
			put(w.in, w.n_split, r16, mp + "a1", rank, D);
			w.hnorm = vec(mp + "norm", vdim, vp);
			w.a2b = vec(mp + "a2.b", H * dim, H * dp, dim, dp);
			const Tensor *s = get2(mp + "a2", H * dim, rank);
			w.a2 = (float *)alloc((size_t)rank * H * dp * sizeof(float));
			if (rc) return;
			TgPack q = pack_of(dev + s->off, s->f32, rank, rank, H * dim);
			q.rows = rank;
			q.cols = H * dp;
			q.g = q.gp = rank;
			q.kg = dim;
			q.kgp = dp;
			q.transpose = 1;
			tg_launch_unpack_f32(w.a2, H * dp, q, n->stream);
		} else if (m.kind == TG_MIX_DELTA) {
			const int G = m.kv_heads, ch = delta_channels(m);
			int d = D, d2 = D;
			m.rank = m.gate_rank = 0;
			get(mp + "a1", {&m.rank, &d});
			get(mp + "g1", {&m.gate_rank, &d2});
			if (rc) return;
			const int rg = tg_up(m.gate_rank, 64), ra = tg_up(m.rank, 16), h16 = tg_up(H, 16);
			w.n_split = ch + rg;
			w.in = mat(w.n_split + h16 + ra, Dp);
			put(w.in, 0, G * dp, mp + "q", G * dim, D, dim, dp);
			put(w.in, G * dp, G * dp, mp + "k", G * dim, D, dim, dp);
			put(w.in, 2 * G * dp, H * vp, mp + "v", H * vdim, D, vdim, vp);
			put(w.in, ch, rg, mp + "g1", m.gate_rank, D);
			put(w.in, w.n_split, h16, mp + "b", H, D);
			put(w.in, w.n_split + h16, ra, mp + "a1", m.rank, D);
			w.conv = (float *)alloc((size_t)m.taps * ch * sizeof(float));
			w.a2 = (float *)alloc((size_t)m.rank * H * dp * sizeof(float));
			w.g2t = (float *)alloc((size_t)m.gate_rank * H * vp * sizeof(float));
			if (rc) return;
			put_transposed(w.conv, ch, G * dp, mp + "q.conv", G * dim, m.taps, dim, dp);
			put_transposed(w.conv + G * dp, ch, G * dp, mp + "k.conv", G * dim, m.taps, dim, dp);
			put_transposed(w.conv + 2 * G * dp, ch, H * vp, mp + "v.conv", H * vdim, m.taps, vdim, vp);
			put_transposed(w.a2, H * dp, H * dp, mp + "a2", H * dim, m.rank, dim, dp);
			put_transposed(w.g2t, H * vp, H * vp, mp + "g2", H * vdim, m.gate_rank, vdim, vp);
			w.g2 = mat(H * vp, rg);
			put(w.g2, 0, H * vp, mp + "g2", H * vdim, m.gate_rank, vdim, vp);
			w.a2b = vec(mp + "dt_bias", H * dim, H * dp, dim, dp);
			w.a_log = vec(mp + "A_log", H, H);
			w.hnorm = vec(mp + "norm", vdim, vp);
		} else if (m.kind == TG_MIX_ATTN) {
			const int G = m.kv_heads;
			w.n_split = (H + G) * dp;
			w.in = mat(w.n_split, Dp);
			put(w.in, 0, H * dp, mp + "q", H * dim, D, dim, dp);
			put(w.in, H * dp, G * dp, mp + "k", G * dim, D, dim, dp);
			w.in_b = vec(mp + "q.b", H * dim, H * dp, dim, dp, 0.0f, (float *)alloc((size_t)w.n_split * sizeof(float)));
			vec(mp + "k.b", G * dim, G * dp, dim, dp, 0.0f, w.in_b + H * dp);
		} else {
			const int R = m.rank, Rp = tg_up(R, 64), h16 = tg_up(H, 16);
			if (m.q_rank) {
				const int Qp = tg_up(m.q_rank, 64), rp = m.rotp(), rd = m.rot_dim;
				w.in = mat(Qp + Rp + rp, Dp);
				put(w.in, 0, Qp, mp + "dq", m.q_rank, D);
				put_part(w.in, Qp, Rp, mp + "dkv", R + rd, D, 0, R);
				put_part(w.in, Qp + Rp, rp, mp + "dkv", R + rd, D, R, rd);
				w.qnorm = vec(mp + "dq.norm", m.q_rank, Qp);
				w.uq = mat(H * (dp + rp), Qp);
				for (int h = 0; h < H && !rc; h++) {
					put_part(w.uq, h * (dp + rp), dp, mp + "uq", H * (dim + rd), m.q_rank, h * (dim + rd), dim);
					put_part(w.uq, h * (dp + rp) + dp, rp, mp + "uq", H * (dim + rd), m.q_rank, h * (dim + rd) + dim, rd);
				}
			} else {
				w.n_split = H * dp;
				w.in = mat(w.n_split + Rp + h16, Dp);
				put(w.in, 0, H * dp, mp + "q", H * dim, D, dim, dp);
				put(w.in, w.n_split, Rp, mp + "dkv", R, D);
				put(w.in, w.n_split + Rp, h16, mp + "g", H, D);
			}
			w.hnorm = vec(mp + "dkv.norm", R, Rp);
			w.uk = mat(H * dp, Rp);
			put(w.uk, 0, H * dp, mp + "uk", H * dim, R, dim, dp);
			w.uv = mat(H * vp, Rp);
			put(w.uv, 0, H * vp, mp + "uv", H * vdim, R, vdim, vp);
			w.uk_t = mat(H * Rp, dp);
			const Tensor *s = get2(mp + "uk", H * dim, R);
			if (rc) return;
			for (int h = 0; h < H; h++) {
				TgPack q = pack_of(dev + s->off + (size_t)h * dim * R * (s->f32 ? 4 : 2), s->f32, R, R, dim);
				q.rows = Rp;
				q.cols = dp;
				q.g = R;
				q.gp = Rp;
				q.kg = dim;
				q.kgp = dp;
				q.transpose = 1;
				q.frag_off = h * Rp / 16;
				tg_launch_pack(w.uk_t, n->dt, q, n->stream);
			}
		}
		w.out = mat(tg_up(D, 64), ko);
		put(w.out, 0, w.out.n, mp + "o", D, H * vdim, 0, 0, vdim, vp);
		if (n->cfg.norm == TG_NORM_RMS) w.n1b = norm(p + "norm1b");
		if (!lc.mlp) return;
		w.n2 = norm(p + "norm2");
		if (n->cfg.norm == TG_NORM_RMS) w.n2b = norm(p + "norm2b");
		if (lc.mlp == TG_FF_DENSE) {
			w.gate_up = mat(lc.moe.ffp(), Dp);
			put(w.gate_up, 0, w.gate_up.n, p + "mlp.up", lc.moe.ff, D);
			w.down = mat(Dp, lc.moe.ffp());
			put(w.down, 0, Dp, p + "mlp.down", D, lc.moe.ff);
			return;
		}
		const int E = lc.moe.experts, ff = lc.moe.ff, fp = lc.moe.ffp();
		const std::string fpfx = p + "mlp.";
		w.router = mat(tg_up(E, 16), Dp);
		put(w.router, 0, w.router.n, fpfx + "router", E, D);
		w.correction = vec(fpfx + "correction", E, E);
		w.gate_up = mat(E * 2 * fp, Dp);
		w.down = mat(E * Dp, fp);
		for (int e = 0; e < E && !rc; e++) {
			const std::string ep = fpfx + "e" + std::to_string(e) + ".";
			put(w.gate_up, 0, fp, ep + "gate", ff, D, 0, 0, 0, 0, 2, e * 2 * fp / 16);
			put(w.gate_up, 0, fp, ep + "up", ff, D, 0, 0, 0, 0, 2, e * 2 * fp / 16 + 1);
			put(w.down, 0, Dp, ep + "down", D, ff, 0, 0, 0, 0, 1, e * Dp / 16);
		}
	}
};

int parse_header(const TgJson &h, size_t data_bytes, std::map<std::string, Tensor> *out) {
	for (const auto &kv : h.members) {
		if (kv.first == "__metadata__") continue;
		Tensor t;
		const TgJson *d = member(&kv.second, "dtype"), *s = member(&kv.second, "shape"), *o = member(&kv.second, "data_offsets");
		if (!d || !s || !o || o->items.size() != 2) return bad("model.safetensors: entry '" + kv.first + "' is not a tensor");
		size_t elem;
		if (d->str == "BF16") { t.f32 = 0; elem = 2; }
		else if (d->str == "F32") { t.f32 = 1; elem = 4; }
		else if (d->str == "I32") { t.f32 = 2; elem = 4; }
		else return bad("model.safetensors: '" + kv.first + "' has the unsupported type " + d->str);
		double n = 1;
		for (const TgJson &x : s->items) {
			if (!(x.num >= 1 && x.num < 1e12)) return bad("model.safetensors: '" + kv.first + "' has a bad shape");
			t.shape.push_back((long long)x.num);
			n *= x.num;
		}
		const double a = o->items[0].num, b = o->items[1].num;
		if (!(a >= 0 && b >= a && b <= (double)data_bytes) || b - a != n * (double)elem)
			return tg_fail(TG_ERR_FILE_SHORT, "model.safetensors: the data of '" + kv.first + "' lie outside the file or do not fit its shape");
		t.off = (size_t)a;
		t.bytes = (size_t)(b - a);
		(*out)[kv.first] = t;
	}
	return TG_OK;
}

int read_text(const std::string &path, std::string *out) {
	FILE *f = fopen(path.c_str(), "rb");
	if (!f) return tg_fail(TG_ERR_FILE_OPEN, "Could not open file. (" + path + ")");
	char buf[65536];
	size_t got;
	while ((got = fread(buf, 1, sizeof(buf), f)) > 0) out->append(buf, got);
	fclose(f);
	return TG_OK;
}

int load_weights(TgNet *n, const std::string &path) {
	const int fd = open(path.c_str(), O_RDONLY);
	if (fd < 0) return tg_fail(TG_ERR_FILE_OPEN, "Could not open file. (" + path + ")");
	struct stat st;
	if (fstat(fd, &st) != 0 || st.st_size < 8) {
		close(fd);
		return tg_fail(TG_ERR_FILE_SHORT, "model.safetensors is too short");
	}
	const size_t size = (size_t)st.st_size;
	const uint8_t *map = (const uint8_t *)mmap(nullptr, size, PROT_READ, MAP_PRIVATE, fd, 0);
	close(fd);
	if (map == MAP_FAILED) return tg_fail(TG_ERR_FILE_OPEN, "Could not open file. (mmap)");
	Loader ld;
	ld.n = n;
	auto run = [&]() -> int {
		uint64_t hl;
		memcpy(&hl, map, 8);
		if (hl > size - 8) return tg_fail(TG_ERR_FILE_SHORT, "model.safetensors is shorter than its header");
		TgJson h;
		std::string err;
		if (!TgJson::parse((const char *)map + 8, hl, &h, &err)) return bad("model.safetensors: " + err);
		const size_t bytes = size - 8 - hl;
		if (int rc = parse_header(h, bytes, &ld.t)) return rc;
		ld.host = map + 8 + hl;
		if (hipMalloc((void **)&ld.dev, std::max<size_t>(bytes, 16)) != hipSuccess) return tg_fail(TG_ERR_HIP, "hipMalloc of the file image failed");
		if (int rc = tg_stage_image(ld.dev, bytes, [&](void *dst, size_t off, size_t len) -> int {
			    memcpy(dst, ld.host + off, len);
			    return TG_OK;
		    }))
			return rc;
		const int D = n->cfg.width, Dp = n->cfg.wp(), V = n->cfg.vocab;
		const Tensor *e = ld.get2("embed", V, D);
		if (ld.rc) return ld.rc;
		if (e->f32) return bad("model.safetensors: 'embed' must be bfloat16");
		n->embed = ld.alloc((size_t)V * Dp * 2);
		if (ld.rc) return ld.rc;
		TG_HIP(hipMemsetAsync(n->embed, 0, (size_t)V * Dp * 2, n->stream));
		TG_HIP(hipMemcpy2DAsync(n->embed, (size_t)Dp * 2, ld.dev + e->off, (size_t)D * 2, (size_t)D * 2, (size_t)V, hipMemcpyDeviceToDevice, n->stream));
		n->fin = ld.norm("final.norm");
		n->head = ld.mat(tg_up(V, 16), Dp);
		ld.put(n->head, 0, n->head.n, "head", V, D);
		n->w.resize(n->cfg.layers.size());
		for (size_t l = 0; l < n->cfg.layers.size() && !ld.rc; l++)
			if (n->cfg.layers[l].weights_of < 0) ld.layer((int)l);
		for (TgNetLayerCfg &lc : n->cfg.layers)
			if (lc.weights_of >= 0) lc.mix.rank = n->cfg.layers[(size_t)lc.weights_of].mix.rank;
		if (ld.rc) return ld.rc;
		TG_HIP(hipGetLastError());
		TG_HIP(hipStreamSynchronize(n->stream));
		return TG_OK;
	};
	const int rc = run();
	if (rc) (void)hipStreamSynchronize(n->stream);
	if (ld.dev) (void)hipFree(ld.dev);
	munmap((void *)map, size);
	return rc;
}

// ---- shared pieces of the two forwards ---------------------------------------------------------------------------------------
int frag_k(int dt) { return dt == TG_DT_BF16 ? 32 : 16; }
long long frags(int dt, int n, int k) { return (long long)(n / 16) * (k / frag_k(dt)); }

// (r: the layer run whose state it works on)
TgGla gla_of(const TgNet *n, int l, TgNetSeq *q, int r) {
	const TgMixerCfg &m = n->cfg.layers[(size_t)l].mix;
	const LayerW &w = n->lw(l);
	TgGla g;
	g.heads = m.heads;
	g.dim = m.dim;
	g.dimp = m.dimp();
	g.vdim = m.vdim;
	g.vdimp = m.vdimp();
	g.rank = m.rank;
	g.qscale = 1.0f / sqrtf((float)m.dim);
	g.inv_tau = 1.0f / m.tau;
	g.eps = n->cfg.eps;
	g.a2 = w.a2;
	g.a2b = w.a2b;
	g.norm = w.hnorm;
	g.state = q ? (float *)q->state[(size_t)r] : nullptr;
	g.a_log = w.a_log;
	g.group = m.kind == TG_MIX_DELTA ? m.heads / m.kv_heads : 1;
	return g;
}

TgDelta delta_of(const TgNet *n, int l, TgNetSeq *q, int r) {
	const TgMixerCfg &m = n->cfg.layers[(size_t)l].mix;
	const LayerW &w = n->lw(l);
	TgDelta d;
	d.g = gla_of(n, l, q, r);
	d.taps = m.taps;
	d.channels = delta_channels(m);
	d.conv = w.conv;
	d.ring = q ? d.g.state + (size_t)m.heads * m.dimp() * m.vdimp() : nullptr;
	d.g2 = w.g2t;
	d.gate_rank = m.gate_rank;
	return d;
}

TgVec vec_of(const TgNet *n, const TgMat &w) {
	TgVec v;
	memset(&v, 0, sizeof(v));
	v.W = w.w;
	v.kfrags = w.k / frag_k(n->dt);
	v.ntiles = w.n / 16;
	v.nz = 1;
	v.ksplit = 1;
	v.eps = n->cfg.eps;
	return v;
}
void norm_prologue(const TgNet *n, TgVec *v, const Norm &nm) {
	v->nw = nm.w;
	v->nb = nm.b;
	v->alpha = nm.alpha;
	v->mult = n->cfg.residual_mult;
	v->width = n->cfg.width;
	v->embed_scale = n->cfg.embed_scale;
}
int norm_kind(const TgNet *n) { return n->cfg.norm == TG_NORM_RMS ? TG_VP_RMS : TG_VP_DYT; }

// Latent attention of one token: keys per workgroup and the number of parts for a context of ctx keys.
void latent_parts(int ctx, int *chunk, int *nb) {
	// As many parts of one tile as a prologue merges; longer contexts need a fold, whose bytes (a partial sum is as large as
	// 32 keys with 16 heads) bound the number of parts from above.
	*chunk = TG_LATENT_TILE;
	if (ctx > TG_LATENT_TILE * TG_LATENT_MAX_PARTS) {
		const int want = (ctx + TG_LATENT_MAX_BLOCKS - 1) / TG_LATENT_MAX_BLOCKS;
		*chunk = std::max(2 * TG_LATENT_TILE, tg_up(want, TG_LATENT_TILE));
	}
	*nb = (ctx + *chunk - 1) / *chunk;
}
// Grouped rows: as many parts as the output product merges in its prologue, of two tiles at most; more keys go to more parts that
// meet in a launch of their own.
void group_parts(int ctx, int heads, int *chunk, int *nb) {
	const bool merge = ctx <= 2 * TG_LATENT_TILE * TG_VEC_MERGE_MAX && heads <= TG_VEC_MERGE_HEADS_MAX;
	const int parts = merge ? TG_VEC_MERGE_MAX : 64;
	*chunk = tg_up(std::max((ctx + parts - 1) / parts, 1), TG_LATENT_TILE);
	*nb = (ctx + *chunk - 1) / *chunk;
}

}  // namespace

bool tg_net_known(const std::string &arch) {
	for (const Arch &a : ARCHS)
		if (arch == a.name) return true;
	return false;
}

int tg_net_open(const char *dir, int dt, int n_cu, hipStream_t s, TgNet **out) {
	if (dt != TG_DT_BF16 && dt != TG_DT_F32) return bad("unknown number format");
	std::string text, err;
	if (int rc = read_text(std::string(dir) + "/config.json", &text)) return rc;
	TgJson j;
	if (!TgJson::parse(text.data(), text.size(), &j, &err)) return bad("config.json: " + err);
	const TgJson *a = member(&j, "architecture");
	if (!a || a->kind != TgJson::String) return bad("config.json names no 'architecture'");
	TgNet *n = new TgNet();
	n->dt = dt;
	n->n_cu = n_cu;
	n->stream = s;
	n->cfg.arch = a->str;
	int rc = tg_fail(TG_ERR_UNSUPPORTED_SHAPE, "unknown architecture '" + a->str + "'");
	for (const Arch &k : ARCHS)
		if (a->str == k.name) rc = k.parse(j, &n->cfg);
	for (const TgNetLayerCfg &l : n->cfg.layers)
		if (!rc && l.mix.kind == TG_MIX_LATENT && tg_latent_step_lds(tg_up(l.mix.rank, 64) + l.mix.rotp(), dt) > TG_LATENT_LDS_MAX)
			rc = tg_fail(TG_ERR_UNSUPPORTED_SHAPE, "kv_rank " + std::to_string(l.mix.rank) + " does not fit the LDS in this number format");
	if (!rc) rc = load_weights(n, std::string(dir) + "/model.safetensors");
	if (rc) {
		tg_net_free(n);
		return rc;
	}
	*out = n;
	return TG_OK;
}

void tg_net_free(TgNet *n) {
	if (!n) return;
	for (void *p : n->owned) (void)hipFree(p);
	delete n;
}

const TgNetCfg &tg_net_cfg(const TgNet *n) { return n->cfg; }
int tg_net_dtype(const TgNet *n) { return n->dt; }
int tg_net_vocab_padded(const TgNet *n) { return n->head.n; }
int tg_net_head_blocks(const TgNet *n) { return tg_vec_blocks(vec_of(n, n->head), TG_VE_LOGITS); }

void tg_net_step_cost(const TgNet *n, double *bytes, int *launches) {
	double b = (double)n->head.n * n->head.k;
	int k = 1;
	for (const int l : n->cfg.runs) {
		const TgNetLayerCfg &c = n->cfg.layers[(size_t)l];
		const LayerW &w = n->lw(l);
		b += (double)w.in.n * w.in.k + (double)w.out.n * w.out.k;
		k += 3;
		if (c.mix.kind == TG_MIX_LATENT) {
			b += (double)w.uk_t.n * w.uk_t.k + (double)w.uv.n * w.uv.k + (double)w.uq.n * w.uq.k;
			k += c.mix.q_rank ? 3 : 2;
		}
		if (c.mlp == TG_FF_DENSE) {
			b += 2.0 * c.moe.ffp() * n->cfg.wp();
			k += 2;
		} else if (c.mlp) {
			b += (double)w.router.n * w.router.k + (double)c.moe.top * 3.0 * c.moe.ffp() * n->cfg.wp();
			k += 3;
		}
	}
	*bytes = b * (double)tg_dt_bytes(n->dt);
	*launches = k;
}

// ---- sequence state ------------------------------------------------------------------------------------------------------------
int tg_net_seq_create(TgNet *n, int capacity, TgNetSeq **out) {
	TgNetSeq *q = new TgNetSeq();
	q->net = n;
	q->capacity = capacity;
	const int R = (int)n->cfg.runs.size(), Dp = n->cfg.wp();
	auto fail = [&](const char *what) {
		tg_net_seq_free(q);
		return tg_fail(TG_ERR_HIP, std::string("session allocation failed: ") + what);
	};
	std::map<std::pair<int, double>, TgRot> tables;
	size_t yin = 0, mix = 0, qp = 0, qq = 0, gate = 0, lg = 0, u = 0, top = 1, acc = 0, ml = 0, facc = 0, pa = 1, pb = 1;
	for (int r = 0; r < R; r++) {
		const int l = n->cfg.runs[(size_t)r];
		const TgNetLayerCfg &c = n->cfg.layers[(size_t)l];
		const TgMixerCfg &m = c.mix;
		const LayerW &w = n->lw(l);
		yin = std::max(yin, (size_t)w.in.n);
		mix = std::max(mix, (size_t)w.out.k);
		pa = std::max(pa, (size_t)tg_vec_ksplit(w.out.n / 16, 1, w.out.k / frag_k(n->dt), n->n_cu));
		size_t bytes;
		TgRot rot = {nullptr, 0, 0};
		if (m.rot_dims) {
			TgRot &t = tables[{m.rot_dims, m.rot_base}];
			if (!t.table) {
				void *p = nullptr;
				if (hipMalloc(&p, (size_t)capacity * (m.rot_dims / 2) * sizeof(float2)) != hipSuccess) return fail("rotary table");
				q->tables.push_back(p);
				tg_launch_rot_table((float2 *)p, capacity, m.rot_dims, m.rot_base, n->stream);
				t.table = (const float2 *)p;
				t.dims = m.rot_dims;
			}
			rot = t;
			rot.half_layout = m.kind == TG_MIX_ATTN;
		}
		q->rot.push_back(rot);
		if (m.kind == TG_MIX_LATENT || m.kind == TG_MIX_ATTN) {
			const size_t G = m.kind == TG_MIX_ATTN ? (size_t)m.kv_heads : 1, Vp = m.kind == TG_MIX_ATTN ? (size_t)m.dimp() : (size_t)tg_up(m.rank, 64);
			const size_t h16 = G * (size_t)tg_up(m.heads / (int)G, 16);
			bytes = (size_t)capacity * G * (Vp + (size_t)m.rotp()) * tg_dt_bytes(n->dt);
			if (m.kind == TG_MIX_LATENT) qp = std::max(qp, (size_t)m.heads * Vp);
			qq = std::max(qq, (size_t)w.uq.n);
			acc = std::max(acc, (size_t)TG_LATENT_MAX_BLOCKS * h16 * Vp);
			ml = std::max(ml, (size_t)TG_LATENT_MAX_BLOCKS * h16 * 2);
			facc = std::max(facc, h16 * Vp);
		} else {
			bytes = (size_t)m.heads * m.dimp() * m.vdimp() * sizeof(float);
			if (m.kind == TG_MIX_DELTA) bytes += (size_t)m.taps * delta_channels(m) * sizeof(float);
			gate = std::max(gate, (size_t)value_width(m));
		}
		void *p = nullptr;
		if (hipMalloc(&p, bytes) != hipSuccess) return fail("layer state");
		q->state.push_back(p);
		// (a tile of the latent cache is read whole, its rows behind the sequence with weight 0: they must hold numbers)
		if (hipMemset(p, 0, bytes) != hipSuccess) return fail("layer state");
		q->state_bytes.push_back(bytes);
		if (c.mlp == TG_FF_DENSE) {
			u = std::max(u, (size_t)c.moe.ffp());
			pb = std::max(pb, (size_t)tg_vec_ksplit(Dp / 16, 1, c.moe.ffp() / frag_k(n->dt), n->n_cu));
		} else if (c.mlp) {
			lg = std::max(lg, (size_t)w.router.n);
			u = std::max(u, (size_t)c.moe.top * c.moe.ffp());
			top = std::max(top, (size_t)c.moe.top);
			pb = std::max(pb, (size_t)c.moe.top * tg_vec_ksplit(Dp / 16, c.moe.top, c.moe.ffp() / frag_k(n->dt), n->n_cu));
		}
	}
	size_t off = 0;
	std::vector<std::pair<void **, size_t>> parts;
	auto want = [&](void **p, size_t elems) {
		parts.emplace_back(p, off);
		off += (elems * 4 + 255) / 256 * 256;
	};
	want((void **)&q->xr, (size_t)(2 * R + 1) * Dp);
	want((void **)&q->yin, yin);
	want((void **)&q->pend_a, pa * Dp);
	want((void **)&q->pend_b, pb * Dp);
	want((void **)&q->hx, (size_t)Dp);
	want((void **)&q->mix, mix);
	want((void **)&q->qp, qp);
	want((void **)&q->qq, qq);
	want((void **)&q->gate, gate);
	want((void **)&q->logits, lg);
	want((void **)&q->u, u);
	want((void **)&q->wgt, top);
	want((void **)&q->sel, top);
	want((void **)&q->acc, acc);
	want((void **)&q->ml, ml);
	want((void **)&q->facc, facc);
	want((void **)&q->fml, facc ? facc : 1);
	if (hipMalloc(&q->ws, off) != hipSuccess) return fail("step buffers");
	for (auto &p : parts) *p.first = (char *)q->ws + p.second;
	if (hipMemset(q->ws, 0, off) != hipSuccess) return fail("step buffers");
	*out = q;
	return tg_net_seq_reset(q);
}

int tg_net_seq_reset(TgNetSeq *q) {
	// Latent rows need no clearing: a row is written before it is read.  Recurrent state starts at zero.
	for (size_t r = 0; r < q->state.size(); r++) {
		const int kind = q->net->cfg.layers[(size_t)q->net->cfg.runs[r]].mix.kind;
		if (kind == TG_MIX_GLA || kind == TG_MIX_DELTA) TG_HIP(hipMemset(q->state[r], 0, q->state_bytes[r]));
	}
	q->tap_rows = 0;
	return TG_OK;
}

void tg_net_seq_release_workspace(TgNetSeq *q) {
	if (q->pf) (void)hipFree(q->pf);
	q->pf = nullptr;
	q->pf_bytes = 0;
	q->taps = nullptr;
	q->tap_rows = 0;
}

void tg_net_seq_free(TgNetSeq *q) {
	if (!q) return;
	for (void *p : q->state)
		if (p) (void)hipFree(p);
	for (void *p : q->tables) (void)hipFree(p);
	if (q->ws) (void)hipFree(q->ws);
	tg_net_seq_release_workspace(q);
	delete q;
}

// ---- one token -------------------------------------------------------------------------------------------------------------------
namespace {

// One decode step: the launches of a mixer and of a feed-forward, and the residual stream between them (x, and parts that the next
// norm adds to it).
struct Step {
	TgNetSeq *q;
	const TgHead &hd;
	int pos, host_pos, pos_bound;  // host_pos: the position, or -1 where the kernels read the counter
	TgNet *n = q->net;
	const TgNetCfg &c = n->cfg;
	const int Dp = c.wp(), dt = n->dt;
	hipStream_t s = n->stream;
	const float *x = nullptr, *pend = nullptr, *post = nullptr;
	int nparts = 0;

	// a product whose prologue norms the residual stream; x_out: where the stream goes
	TgVec normed(const TgMat &w, const Norm &nm, float *x_out) {
		TgVec v = vec_of(n, w);
		norm_prologue(n, &v, nm);
		if (x) {
			v.x = x;
		} else {
			v.embed = n->embed;
			v.embed_ld = Dp;
			v.vocab = c.vocab;
			v.ctr = hd.ctr;
		}
		v.pend = pend;
		v.nparts = nparts;
		v.pend_stride = Dp;
		v.post = post;
		v.x_out = x_out;
		x = x_out;
		return v;
	}
	// what a sublayer leaves for the next norm
	void leave(const float *parts, int count, const Norm &after) {
		pend = parts;
		nparts = count;
		post = after.w;
	}

	void gla(int l, int r, TgVec o) {
		const TgMixerCfg &m = c.layers[(size_t)l].mix;
		const LayerW &w = n->lw(l);
		tg_launch_gla_step(gla_of(n, l, q, r), q->yin, row_k_off(m), row_v_off(m), w.n_split, q->mix, s);
		o.gate = q->yin + row_g_off(m);
		head_norm(m, w, o);
	}
	void delta(int l, int r, TgVec o) {
		const TgMixerCfg &m = c.layers[(size_t)l].mix;
		const LayerW &w = n->lw(l);
		tg_launch_delta_step(delta_of(n, l, q, r), q->yin, delta_channels(m), w.n_split, w.n_split + tg_up(m.heads, 16), hd.ctr, host_pos, q->mix, q->gate,
		                     s);
		o.gate = q->gate;
		o.gate_sigmoid = 1;
		head_norm(m, w, o);
	}
	void head_norm(const TgMixerCfg &m, const LayerW &w, TgVec &o) {
		o.nw = w.hnorm;
		o.vdim = m.vdim;
		o.vdimp = m.vdimp();
		o.heads16 = m.heads;
		tg_launch_vec(o, dt, TG_VP_HEADNORM, TG_VE_STORE, s);
	}
	TgLatentStep shared_rows(int l, int r) {
		const TgMixerCfg &m = c.layers[(size_t)l].mix;
		TgLatentStep t;
		memset(&t, 0, sizeof(t));
		t.rot = q->rot[(size_t)r];
		t.rotp = m.rotp();
		t.eps = c.eps;
		t.scale = m.scale;
		t.window = m.window;
		t.cache = q->state[(size_t)r];
		t.ctr = hd.ctr;
		t.host_pos = host_pos;
		t.part_acc = q->acc;
		t.part_ml = q->ml;
		return t;
	}
	void latent(int l, int r, const TgVec &o) {
		const TgMixerCfg &m = c.layers[(size_t)l].mix;
		const LayerW &w = n->lw(l);
		const int Rp = tg_up(m.rank, 64), h16 = tg_up(m.heads, 16), Qp = tg_up(m.q_rank, 64), qs = m.dimp() + m.rotp();
		const float *qv = q->yin, *kv = q->yin + w.n_split, *gate = kv + Rp;
		if (m.q_rank) {
			TgVec u = vec_of(n, w.uq);
			u.x = q->yin;
			u.nw = w.qnorm;
			u.width = m.q_rank;
			u.y = q->qq;
			tg_launch_vec(u, dt, TG_VP_RMS, TG_VE_STORE, s);
			qv = q->qq;
			kv = q->yin + Qp;
			gate = nullptr;
		}
		TgVec a = vec_of(n, w.uk_t);
		a.ntiles = Rp / 16;
		a.nz = m.heads;
		a.zfrags = frags(dt, Rp, m.dimp());
		a.x = qv;
		a.x_zstride = qs;
		a.y = q->qp;
		a.y_zstride = Rp;
		tg_launch_vec(a, dt, TG_VP_PLAIN, TG_VE_STORE, s);
		TgLatentStep t = shared_rows(l, r);
		t.groups = 1;
		t.heads = m.heads;
		t.rank = m.rank;
		t.rankp = Rp;
		t.rot_size = m.rot_dim;
		t.q = q->qp;
		t.q_stride = Rp;
		t.qr = qv + m.dimp();
		t.qr_stride = qs;
		t.kv = kv;
		t.kr = kv + Rp;
		t.norm = w.hnorm;
		latent_parts(std::min(pos_bound + 1, m.window), &t.chunk, &t.nb);
		tg_launch_latent_step(t, dt, s);
		const bool fold = t.nb > TG_LATENT_MAX_PARTS;
		if (fold) tg_launch_latent_fold(q->acc, q->ml, t.nb, h16, Rp, q->facc, q->fml, s);
		TgVec b = vec_of(n, w.uv);
		b.ntiles = m.vdimp() / 16;
		b.nz = m.heads;
		b.zfrags = frags(dt, m.vdimp(), Rp);
		b.part_acc = fold ? q->facc : q->acc;
		b.part_ml = fold ? q->fml : q->ml;
		b.nmerge = fold ? 1 : t.nb;
		b.heads16 = h16;
		b.x_zstride = Rp;
		b.gate = gate;
		b.y = q->mix;
		b.y_zstride = m.vdimp();
		tg_launch_vec(b, dt, TG_VP_MERGE, gate ? TG_VE_GATE : TG_VE_STORE, s);
		tg_launch_vec(o, dt, TG_VP_PLAIN, TG_VE_STORE, s);
	}
	void attention(int l, int r, TgVec o) {
		const TgMixerCfg &m = c.layers[(size_t)l].mix;
		const int dp = m.dimp();
		const float *k = q->yin + m.heads * dp;
		TgLatentStep t = shared_rows(l, r);
		t.groups = m.kv_heads;
		t.heads = m.heads / m.kv_heads;
		t.rank = m.dim;
		t.rankp = dp;
		t.rot_size = t.q_zero = m.rot_dims;
		t.q = t.qr = q->yin;
		t.q_stride = t.qr_stride = dp;
		t.kv = t.kr = k;
		t.kv_stride = t.kr_stride = dp;
		group_parts(std::min(pos_bound + 1, m.window), m.heads, &t.chunk, &t.nb);
		tg_launch_latent_step(t, dt, s);
		if (t.nb <= TG_VEC_MERGE_MAX && m.heads <= TG_VEC_MERGE_HEADS_MAX) {
			o.part_acc = q->acc;
			o.part_ml = q->ml;
			o.nmerge = t.nb;
			o.heads16 = t.groups * tg_up(t.heads, 16);
			o.group = t.heads;
			o.heads = m.heads;
			o.vdimp = o.x_zstride = dp;
			tg_launch_vec(o, dt, TG_VP_MERGE_HEADS, TG_VE_STORE, s);
			return;
		}
		tg_launch_latent_finish(q->acc, q->ml, t.nb, t.groups, t.heads, dp, q->mix, dp, s);
		tg_launch_vec(o, dt, TG_VP_PLAIN, TG_VE_STORE, s);
	}

	void experts(int l, float *x_out) {
		const LayerW &w = n->lw(l);
		const TgMoeCfg &e = c.layers[(size_t)l].moe;
		TgVec r = normed(w.router, w.n2, x_out);
		r.h_out = q->hx;
		r.y = q->logits;
		tg_launch_vec(r, dt, norm_kind(n), TG_VE_STORE, s);
		TgVec g = vec_of(n, w.gate_up);
		g.ntiles = 2 * e.ffp() / 16;
		g.nz = e.top;
		g.zfrags = frags(dt, 2 * e.ffp(), Dp);
		g.x = q->hx;
		g.logits = q->logits;
		g.correction = w.correction;
		g.experts = e.experts;
		g.top = e.top;
		g.rscale = e.scale;
		g.sel = q->sel;
		g.wgt = q->wgt;
		g.y = q->u;
		g.y_zstride = e.ffp();
		tg_launch_vec(g, dt, TG_VP_EXPERT, TG_VE_SWIGLU, s);
		TgVec d = vec_of(n, w.down);
		d.ntiles = Dp / 16;
		d.nz = e.top;
		d.zfrags = frags(dt, Dp, e.ffp());
		d.ksplit = tg_vec_ksplit(d.ntiles, d.nz, d.kfrags, n->n_cu);
		d.x = q->u;
		d.x_zstride = e.ffp();
		d.sel = q->sel;
		d.wgt = q->wgt;
		d.y = q->pend_b;
		d.part_stride = Dp;
		d.y_zstride = d.ksplit * Dp;
		tg_launch_vec(d, dt, TG_VP_PLAIN, TG_VE_WEIGHTED, s);
		leave(q->pend_b, e.top * d.ksplit, w.n2b);
	}
	void dense(int l, float *x_out) {
		const LayerW &w = n->lw(l);
		TgVec u = normed(w.gate_up, w.n2, x_out);
		u.y = q->u;
		tg_launch_vec(u, dt, norm_kind(n), TG_VE_GELU, s);
		TgVec d = vec_of(n, w.down);
		d.ksplit = tg_vec_ksplit(d.ntiles, 1, d.kfrags, n->n_cu);
		d.x = q->u;
		d.y = q->pend_b;
		d.part_stride = Dp;
		tg_launch_vec(d, dt, TG_VP_PLAIN, TG_VE_STORE, s);
		leave(q->pend_b, d.ksplit, w.n2b);
	}

	void run() {
		const int R = (int)c.runs.size();
		for (int r = 0; r < R; r++) {
			const int l = c.runs[(size_t)r];
			const TgNetLayerCfg &lc = c.layers[(size_t)l];
			const LayerW &w = n->lw(l);
			TgVec v = normed(w.in, w.n1, q->xr + (size_t)(2 * r) * Dp);
			v.bias = w.in_b;
			v.y = q->yin;
			tg_launch_vec(v, dt, norm_kind(n), TG_VE_STORE, s);
			TgVec o = vec_of(n, w.out);
			o.ksplit = tg_vec_ksplit(o.ntiles, 1, o.kfrags, n->n_cu);
			o.part_stride = Dp;
			o.y = q->pend_a;
			o.x = q->mix;
			switch (lc.mix.kind) {
				case TG_MIX_GLA: gla(l, r, o); break;
				case TG_MIX_DELTA: delta(l, r, o); break;
				case TG_MIX_ATTN: attention(l, r, o); break;
				default: latent(l, r, o); break;
			}
			leave(q->pend_a, o.ksplit, w.n1b);
			float *behind = q->xr + (size_t)(2 * r + 1) * Dp;
			if (lc.mlp == TG_FF_MOE) experts(l, behind);
			else if (lc.mlp == TG_FF_DENSE) dense(l, behind);
		}
		TgVec v = normed(n->head, n->fin, q->xr + (size_t)(2 * R) * Dp);
		v.y = hd.logits;
		v.nout = c.vocab;
		v.blk_val = hd.blk_val;
		v.blk_idx = hd.blk_idx;
		tg_launch_vec(v, dt, norm_kind(n), TG_VE_LOGITS, s);
	}
};

}  // namespace

int tg_net_step(TgNetSeq *q, const TgHead &hd, int pos, bool host_pos, int pos_bound) {
	Step{q, hd, pos, host_pos ? pos : -1, pos_bound}.run();
	q->tap_rows = 0;
	return TG_OK;
}

// ---- many tokens -----------------------------------------------------------------------------------------------------------------
namespace {

struct Arena {
	unsigned char *base = nullptr;
	size_t off = 0;
	template <class P>
	void take(P **p, size_t bytes) {
		*p = base ? (P *)(base + off) : nullptr;
		off += (bytes + 255) / 256 * 256;
	}
};

struct Rows {
	int *ids, *want, *sel, *slot, *row_src, *count, *ntiles;
	int4 *tiles;
	float *x, *low, *rl, *wgt, *lg, *sub;  // sub: a sublayer's output before the norm behind it
	void *h, *in, *mix, *u, *y, *hw, *k, *vt, *qn, *q, *gate;
	unsigned char *gla;
	float *taps;
};

// workspace of one pass of n tokens behind `past`
void rows_layout(const TgNet *n, int rows, int past, int n_want, int tap_rows, Arena *a, Rows *r) {
	const TgNetCfg &c = n->cfg;
	const size_t N = (size_t)rows, Dp = (size_t)c.wp(), eb = tg_dt_bytes(n->dt);
	size_t in = 0, low = 0, mix = 0, gla = 0, k = 0, vt = 0, rl = 0, top = 0, u = 0, cnt = 0, tiles = 0, qn = 0, ql = 0, gate = 0;
	for (size_t l = 0; l < c.layers.size(); l++) {
		const TgNetLayerCfg &lc = c.layers[l];
		const LayerW &w = n->lw((int)l);
		in = std::max(in, (size_t)w.n_split);
		low = std::max(low, (size_t)(w.in.n - w.n_split));
		mix = std::max(mix, (size_t)w.out.k);
		const size_t ctxp = (size_t)tg_up(past + rows - window_start(lc.mix, past), 64);
		if (lc.mix.kind == TG_MIX_GLA) {
			gla = std::max(gla, tg_gla_scratch(gla_of(n, (int)l, nullptr, 0), rows, nullptr, nullptr));
		} else if (lc.mix.kind == TG_MIX_DELTA) {
			gla = std::max(gla, tg_delta_scratch(delta_of(n, (int)l, nullptr, 0), rows, nullptr, nullptr));
			gate = std::max(gate, (size_t)value_width(lc.mix));
		} else if (lc.mix.kind == TG_MIX_ATTN) {
			k = std::max(k, ctxp * (size_t)(lc.mix.kv_heads * lc.mix.dimp()) * eb);
			vt = std::max(vt, ctxp * (size_t)(lc.mix.kv_heads * lc.mix.dimp()) * eb);
		} else {
			k = std::max(k, ctxp * (size_t)w.uk.n * eb);
			vt = std::max(vt, ctxp * (size_t)w.uv.n * eb);
			qn = std::max(qn, (size_t)w.uq.k);
			ql = std::max(ql, (size_t)w.uq.n);
		}
		if (lc.mlp == TG_FF_DENSE) {
			u = std::max(u, N * lc.moe.ffp() * eb);
		} else if (lc.mlp) {
			rl = std::max(rl, (size_t)w.router.n);
			top = std::max(top, (size_t)lc.moe.top);
			u = std::max(u, N * lc.moe.top * lc.moe.ffp() * eb);
			cnt = std::max(cnt, (size_t)((rows + TG_MOE_BLOCK - 1) / TG_MOE_BLOCK) * lc.moe.experts);
			tiles = std::max(tiles, (size_t)tg_moe_max_tiles(rows, lc.moe.experts, lc.moe.top, 32));
		}
	}
	a->take(&r->ids, N * 4);
	a->take(&r->want, (size_t)WANT_ROWS * 4);
	a->take(&r->x, N * Dp * 4);
	a->take(&r->h, N * Dp * eb);
	a->take(&r->in, N * in * eb);
	a->take(&r->low, N * low * 4);
	a->take(&r->mix, N * mix * eb);
	a->take(&r->qn, N * qn * eb);
	a->take(&r->q, N * ql * eb);
	a->take(&r->gate, N * gate * eb);
	a->take(&r->sub, c.norm == TG_NORM_RMS ? N * Dp * 4 : 0);
	a->take(&r->gla, gla);
	a->take(&r->k, k);
	a->take(&r->vt, vt);
	a->take(&r->rl, N * rl * 4);
	a->take(&r->sel, N * top * 4);
	a->take(&r->wgt, N * top * 4);
	a->take(&r->slot, N * top * 4);
	a->take(&r->row_src, N * top * 4);
	a->take(&r->count, cnt * 4);
	a->take(&r->tiles, tiles * 16);
	a->take(&r->ntiles, 4);
	a->take(&r->u, u);
	a->take(&r->y, N * top * Dp * eb);
	const size_t W = (size_t)std::min(n_want, WANT_ROWS);
	a->take(&r->hw, W * Dp * eb);
	a->take(&r->lg, W * (size_t)n->head.n * 4);
	a->take(&r->taps, (size_t)(2 * c.runs.size() + 1) * (size_t)tap_rows * Dp * 4);
}

TgGemm gemm_of(const void *A, int lda, const TgMat &w, int rows) {
	TgGemm g;
	memset(&g, 0, sizeof(g));
	g.A = A;
	g.lda = lda;
	g.W = w.w;
	g.M = rows;
	g.K = w.k;
	g.N = w.n;
	return g;
}

// One pass of a portion.
struct Pass {
	TgNetSeq *q;
	const Rows &r;
	int rows, pos, tap_rows;
	TgNet *n = q->net;
	const TgNetCfg &c = n->cfg;
	const int Dp = c.wp(), dt = n->dt;
	const bool rms = c.norm == TG_NORM_RMS;
	const size_t eb = tg_dt_bytes(dt);
	hipStream_t s = n->stream;
	TgRowsDyt d = {};           // state of the residual stream: what the next row step still adds
	const float *post = nullptr;  // (root mean square norms) weight of the norm behind the sublayer in r.sub; null: nothing waits
	bool embed = true;
	int due[2] = {-1, -1};      // blocks whose residual is complete behind the next row step

	void start() {
		memset(&d, 0, sizeof(d));
		d.x = r.x;
		d.ldx = Dp;
		d.n = rows;
		d.embed = n->embed;
		d.ids = r.ids;
		d.vocab = c.vocab;
		d.mult = c.residual_mult;
	}
	void tap(int b) {
		if (tap_rows && b >= 0) tg_launch_copy(r.taps + (size_t)b * tap_rows * Dp, r.x, (size_t)rows * Dp * sizeof(float), s);
	}
	TgRowsRms rms_rows(const Norm *nm) {
		TgRowsRms k;
		memset(&k, 0, sizeof(k));
		k.x = r.x;
		k.ldx = k.ldo = Dp;
		k.n = rows;
		k.width = c.width;
		k.eps = c.eps;
		k.nw = nm ? nm->w : nullptr;
		return k;
	}
	// the row step: what waits is added to the residual stream, then the norm `nm` of it goes to r.h (null: none)
	void advance(const Norm *nm) {
		if (rms) {
			TgRowsRms k = rms_rows(nm);
			if (embed) {
				k.embed = n->embed;
				k.ids = r.ids;
				k.vocab = c.vocab;
				k.embed_scale = c.embed_scale;
			}
			if (post) {
				k.y = r.sub;
				k.ldy = Dp;
				k.post = post;
			}
			k.out = nm ? r.h : nullptr;
			tg_launch_rows_rms(k, dt, s);
			post = nullptr;
		} else {
			d.out = nm ? r.h : nullptr;
			if (nm) {
				d.alpha = nm->alpha;
				d.nw = nm->w;
				d.nb = nm->b;
			}
			tg_launch_rows_dyt(d, dt, s);
			d.embed = nullptr;
			d.y = nullptr;
		}
		embed = false;
		for (int &b : due) {
			tap(b);
			b = -1;
		}
	}
	bool waiting() const { return rms ? post != nullptr : d.y != nullptr; }

	void gla(int l, int run) {
		const TgMixerCfg &m = c.layers[(size_t)l].mix;
		const LayerW &w = n->lw(l);
		const TgGla ga = gla_of(n, l, q, run);
		TgGlaScratch t;
		tg_gla_scratch(ga, rows, &t, r.gla);
		tg_launch_gla_rows(ga, dt, r.in, w.n_split, row_k_off(m), row_v_off(m), row_g_off(m), r.low, w.in.n - w.n_split, rows, t, r.mix, w.out.k, s);
	}
	void delta(int l, int run) {
		const TgMixerCfg &m = c.layers[(size_t)l].mix;
		const LayerW &w = n->lw(l);
		const TgDelta de = delta_of(n, l, q, run);
		TgGemm g = gemm_of((const unsigned char *)r.in + (size_t)delta_channels(m) * eb, w.n_split, w.g2, rows);
		g.C = r.gate;
		g.ldc = g.n_split = w.g2.n;
		tg_launch_linear(g, dt, TG_GE_STORE, s);
		TgDeltaScratch t;
		tg_delta_scratch(de, rows, &t, r.gla);
		tg_launch_delta_rows(de, dt, r.in, w.n_split, r.low, w.in.n - w.n_split, 0, tg_up(m.heads, 16), r.gate, w.g2.n, rows, pos, t, r.mix, w.out.k, s);
	}
	TgLatentRows tiled(const TgMixerCfg &m, const LayerW &w, int lo) {
		TgLatentRows t;
		memset(&t, 0, sizeof(t));
		t.k = r.k;
		t.vt = r.vt;
		t.ldv = tg_up(pos + rows - lo, 64);
		t.out = r.mix;
		t.ldo = w.out.k;
		t.n = rows;
		t.past = pos - lo;
		t.heads = m.heads;
		t.group = 1;
		t.dimp = m.dimp();
		t.vdimp = m.vdimp();
		t.window = m.window;
		t.scale = m.scale;
		return t;
	}
	void latent(int l, int run) {
		const TgMixerCfg &m = c.layers[(size_t)l].mix;
		const LayerW &w = n->lw(l);
		const int Rp = tg_up(m.rank, 64), Qp = tg_up(m.q_rank, 64), rowp = Rp + m.rotp(), ldl = w.in.n - w.n_split;
		const int lo = window_start(m, pos), ctx = pos + rows - lo;
		unsigned char *cache = (unsigned char *)q->state[(size_t)run];
		TgLatentCacheRows cr;
		memset(&cr, 0, sizeof(cr));
		cr.kv = r.low + Qp;
		cr.kr = r.low + Qp + Rp;
		cr.ld = ldl;
		cr.f32 = 1;
		cr.n = rows;
		cr.past = pos;
		cr.groups = 1;
		cr.rank = m.rank;
		cr.rankp = Rp;
		cr.rot_size = m.rot_dim;
		cr.rotp = m.rotp();
		cr.rot = q->rot[(size_t)run];
		cr.norm = w.hnorm;
		cr.eps = c.eps;
		cr.cache = cache;
		tg_launch_latent_rows(cr, dt, s);
		TgLatentRows t = tiled(m, w, lo);
		if (m.q_rank) {
			TgRowsRms k;
			memset(&k, 0, sizeof(k));
			k.x = r.low;
			k.ldx = ldl;
			k.n = rows;
			k.width = m.q_rank;
			k.eps = c.eps;
			k.nw = w.qnorm;
			k.out = r.qn;
			k.ldo = Qp;
			k.cols = Qp;
			tg_launch_rows_rms(k, dt, s);
			TgGemm u = gemm_of(r.qn, Qp, w.uq, rows);
			u.C = r.q;
			u.ldc = u.n_split = w.uq.n;
			tg_launch_linear(u, dt, TG_GE_STORE, s);
			tg_launch_rot_rows(r.q, w.uq.n, rows, pos, m.dimp(), m.heads, m.dimp() + m.rotp(), cr.rot, dt, s);
			t.q = r.q;
			t.ldq = w.uq.n;
			t.rotp = m.rotp();
			t.kr = cache + ((size_t)lo * rowp + Rp) * eb;
			t.ldkr = rowp;
		} else {
			t.q = r.in;
			t.ldq = w.n_split;
			t.gate = r.low + Rp;
			t.ld_gate = ldl;
		}
		const unsigned char *first = cache + (size_t)lo * rowp * eb;
		TgGemm k = gemm_of(first, rowp, w.uk, ctx);
		k.C = r.k;
		k.ldc = k.n_split = t.ldk = w.uk.n;
		tg_launch_linear(k, dt, TG_GE_STORE, s);
		TgGemm v = gemm_of(first, rowp, w.uv, ctx);
		v.C = r.vt;
		v.ldc = v.rows_out = t.ldv;
		tg_launch_linear(v, dt, TG_GE_TRANS, s);
		tg_launch_latent_attention(t, dt, s);
	}
	void attention(int l, int run) {
		const TgMixerCfg &m = c.layers[(size_t)l].mix;
		const LayerW &w = n->lw(l);
		const int dp = m.dimp(), lo = window_start(m, pos);
		TgLatentCacheRows cr;
		memset(&cr, 0, sizeof(cr));
		cr.kv = cr.kr = (const unsigned char *)r.in + (size_t)m.heads * dp * eb;
		cr.ld = w.n_split;
		cr.kv_stride = cr.kr_stride = dp;
		cr.n = rows;
		cr.past = pos;
		cr.groups = m.kv_heads;
		cr.rank = m.dim;
		cr.rankp = dp;
		cr.rot_size = m.rot_dims;
		cr.rotp = m.rotp();
		cr.rot = q->rot[(size_t)run];
		cr.cache = q->state[(size_t)run];
		tg_launch_latent_rows(cr, dt, s);
		tg_launch_rot_rows(r.in, w.n_split, rows, pos, 0, m.heads, dp, cr.rot, dt, s);
		TgLatentRows t = tiled(m, w, lo);
		TgKeyValues kv;
		kv.cache = cr.cache;
		kv.lo = lo;
		kv.n = pos + rows - lo;
		kv.groups = m.kv_heads;
		kv.dimp = dp;
		kv.rot_size = m.rot_dims;
		kv.rotp = m.rotp();
		kv.k = r.k;
		kv.vt = r.vt;
		kv.ldv = t.ldv;
		tg_launch_key_values(kv, dt, s);
		t.q = r.in;
		t.ldq = w.n_split;
		t.ldk = m.kv_heads * dp;
		t.group = m.heads / m.kv_heads;
		tg_launch_latent_attention(t, dt, s);
	}

	void experts(int l) {
		const LayerW &w = n->lw(l);
		const TgMoeCfg &e = c.layers[(size_t)l].moe;
		TgGemm rt = gemm_of(r.h, Dp, w.router, rows);
		rt.C2 = r.rl;
		rt.ldc2 = w.router.n;
		tg_launch_linear(rt, dt, TG_GE_F32, s);
		TgMoeRoute mr;
		mr.logits = r.rl;
		mr.ld = w.router.n;
		mr.correction = w.correction;
		mr.n = rows;
		mr.experts = e.experts;
		mr.top = e.top;
		const long long per_expert = (long long)rows * e.top / e.experts;
		mr.tile_rows = per_expert >= 128 ? 128 : (per_expert >= 48 ? 64 : 32);
		mr.scale = e.scale;
		mr.sel = r.sel;
		mr.wgt = r.wgt;
		mr.slot = r.slot;
		mr.row_src = r.row_src;
		mr.count = r.count;
		mr.tiles = r.tiles;
		mr.ntiles = r.ntiles;
		tg_launch_moe_route(mr, s);
		TgGemm gu = gemm_of(r.h, Dp, w.gate_up, rows * e.top);
		gu.N = 2 * e.ffp();
		gu.C = r.u;
		gu.ldc = e.ffp();
		gu.tiles = r.tiles;
		gu.ntiles = r.ntiles;
		gu.max_tiles = tg_moe_max_tiles(rows, e.experts, e.top, mr.tile_rows);
		gu.tile_rows = mr.tile_rows;
		gu.row_src = r.row_src;
		gu.group_frags = frags(dt, 2 * e.ffp(), Dp);
		tg_launch_linear(gu, dt, TG_GE_SWIGLU, s);
		TgGemm dn = gemm_of(r.u, e.ffp(), w.down, rows * e.top);
		dn.N = Dp;
		dn.C = r.y;
		dn.ldc = dn.n_split = Dp;
		dn.tiles = gu.tiles;
		dn.ntiles = gu.ntiles;
		dn.max_tiles = gu.max_tiles;
		dn.tile_rows = gu.tile_rows;
		dn.group_frags = frags(dt, Dp, e.ffp());
		tg_launch_linear(dn, dt, TG_GE_STORE, s);
		d.y = r.y;
		d.slot = r.slot;
		d.wgt = r.wgt;
		d.top = e.top;
	}
	void dense(int l) {
		const LayerW &w = n->lw(l);
		TgGemm u = gemm_of(r.h, Dp, w.gate_up, rows);
		u.C = r.u;
		u.ldc = w.gate_up.n;
		tg_launch_linear(u, dt, TG_GE_GELU, s);
		result(r.u, w.gate_up.n, w.down, w.n2b);
	}
	// a sublayer's last product, into the residual stream or to wait for the norm behind it
	void result(const void *a, int lda, const TgMat &w, const Norm &after) {
		TgGemm o = gemm_of(a, lda, w, rows);
		o.C2 = rms ? r.sub : r.x;
		o.ldc2 = Dp;
		o.mult = c.residual_mult;
		tg_launch_linear(o, dt, rms ? TG_GE_F32 : TG_GE_RESID, s);
		post = after.w;
	}

	void run() {
		start();
		const int R = (int)c.runs.size();
		due[0] = 0;
		for (int i = 0; i < R; i++) {
			const int l = c.runs[(size_t)i];
			const TgNetLayerCfg &lc = c.layers[(size_t)l];
			const LayerW &w = n->lw(l);
			advance(&w.n1);
			TgGemm g = gemm_of(r.h, Dp, w.in, rows);
			const int nlow = w.in.n - w.n_split;
			g.C = r.in;
			g.ldc = g.n_split = w.n_split;
			g.C2 = r.low;
			g.ldc2 = nlow;
			g.bias = w.in_b;
			if (nlow > 0 && w.n_split > 0 && nlow <= 64 && rows >= 128) {
				// a few fp32 columns behind the others would start another column of tiles: a product of their own
				TgGemm low = g;
				low.W = (const unsigned char *)w.in.w + frags(dt, w.n_split, w.in.k) * 1024;
				g.N = w.n_split;
				low.N = nlow;
				tg_launch_linear(low, dt, TG_GE_F32, s);
			}
			tg_launch_linear(g, dt, w.n_split ? TG_GE_STORE : TG_GE_F32, s);
			switch (lc.mix.kind) {
				case TG_MIX_GLA: gla(l, i); break;
				case TG_MIX_DELTA: delta(l, i); break;
				case TG_MIX_ATTN: attention(l, i); break;
				default: latent(l, i); break;
			}
			result(r.mix, w.out.k, w.out, w.n1b);
			if (rms) due[0] = 2 * i + 1;
			else tap(2 * i + 1);
			if (lc.mlp) {
				advance(&w.n2);
				if (lc.mlp == TG_FF_DENSE) dense(l);
				else experts(l);
				due[0] = -1;
			}
			due[1] = 2 * i + 2;
		}
		if (waiting()) advance(nullptr);
		for (const int b : due) tap(b);  // (nothing waited)
	}
	// logits of chosen rows
	void wanted(const int *dev_rows, int count, float *lg) {
		if (rms) {
			TgRowsRms k = rms_rows(&n->fin);
			k.n = count;
			k.gather = dev_rows;
			k.out = r.hw;
			tg_launch_rows_rms(k, dt, s);
		} else {
			TgRowsDyt f = d;
			f.n = count;
			f.gather = dev_rows;
			f.y = nullptr;
			f.embed = nullptr;
			f.alpha = n->fin.alpha;
			f.nw = n->fin.w;
			f.nb = n->fin.b;
			f.out = r.hw;
			tg_launch_rows_dyt(f, dt, s);
		}
		TgGemm g = gemm_of(r.hw, Dp, n->head, count);
		g.C2 = lg;
		g.ldc2 = n->head.n;
		tg_launch_linear(g, dt, TG_GE_F32, s);
	}
};

}  // namespace

static int net_pass(TgNetSeq *q, const int32_t *ids, int rows, int pos, const int32_t *want, int n_want, float *logits, const TgHead *hd,
                    int tap_rows) {
	TgNet *n = q->net;
	const TgNetCfg &c = n->cfg;
	const int Dp = c.wp(), dt = n->dt;
	hipStream_t s = n->stream;
	Arena a;
	Rows r;
	rows_layout(n, rows, pos, n_want, tap_rows, &a, &r);
	if (a.off > q->pf_bytes) {
		TG_HIP(hipStreamSynchronize(s));
		tg_net_seq_release_workspace(q);
		TG_HIP(hipMalloc(&q->pf, a.off));
		q->pf_bytes = a.off;
	}
	a.base = (unsigned char *)q->pf;
	a.off = 0;
	rows_layout(n, rows, pos, n_want, tap_rows, &a, &r);
	TG_HIP(hipMemcpyAsync(r.ids, ids, sizeof(int) * (size_t)rows, hipMemcpyHostToDevice, s));
	Pass p{q, r, rows, pos, tap_rows};
	p.run();
	for (int w0 = 0; w0 < n_want; w0 += WANT_ROWS) {
		const int nw = std::min(WANT_ROWS, n_want - w0);
		TG_HIP(hipMemcpyAsync(r.want, want + w0, sizeof(int) * (size_t)nw, hipMemcpyHostToDevice, s));
		p.wanted(r.want, nw, r.lg);
		TG_HIP(hipMemcpy2DAsync(logits + (size_t)w0 * c.vocab, sizeof(float) * (size_t)c.vocab, r.lg, sizeof(float) * (size_t)n->head.n,
		                        sizeof(float) * (size_t)c.vocab, (size_t)nw, hipMemcpyDeviceToHost, s));
	}
	if (hd) {
		TgVec v = vec_of(n, n->head);
		norm_prologue(n, &v, n->fin);
		v.x = r.x + (size_t)(rows - 1) * Dp;
		v.y = hd->logits;
		v.nout = c.vocab;
		v.blk_val = hd->blk_val;
		v.blk_idx = hd->blk_idx;
		tg_launch_vec(v, dt, norm_kind(n), TG_VE_LOGITS, s);
	}
	q->taps = tap_rows ? r.taps : nullptr;
	q->tap_rows = tap_rows;
	TG_HIP(hipGetLastError());
	return TG_OK;
}

int tg_net_rows(TgNetSeq *q, const int32_t *ids, int n, int pos, const int32_t *want, int n_want, float *logits, const TgHead &h, bool taps) {
	int w = 0;
	std::vector<int32_t> rel;
	for (int i = 0; i < n; i += SLICE) {
		const int m = std::min(SLICE, n - i);
		rel.clear();
		const int w0 = w;
		while (w < n_want && want[w] < i + m) rel.push_back(want[w++] - i);
		if (int rc = net_pass(q, ids + i, m, pos + i, rel.data(), (int)rel.size(), logits + (size_t)w0 * q->net->cfg.vocab, i + m == n ? &h : nullptr,
		                      taps && n <= TAP_MAX_ROWS ? n : 0))
			return rc;
		// `rel` and the caller's arrays may be reused as soon as the copies have been made
		TG_HIP(hipStreamSynchronize(q->net->stream));
	}
	return TG_OK;
}

void tg_net_replayed(TgNetSeq *q) { q->tap_rows = 0; }

int tg_net_tap(TgNetSeq *q, int b, float *out, int rows) {
	const TgNetCfg &c = q->net->cfg;
	const size_t Dp = (size_t)c.wp(), D = (size_t)c.width;
	if (q->tap_rows) {
		if (rows != q->tap_rows) return bad("rows must equal the portion's length");
	} else {
		if (rows != 1) return bad("decode taps have one row");
		// without a feed-forward the residual behind the layer is the one behind its mixer
		if (b % 2 == 1 && !c.layers[(size_t)c.runs[(size_t)(b / 2)]].mlp) b += 1;
	}
	const float *src = q->tap_rows ? q->taps + (size_t)b * rows * Dp : q->xr + (size_t)b * Dp;
	TG_HIP(hipMemcpy2D(out, D * 4, src, Dp * 4, D * 4, (size_t)rows, hipMemcpyDeviceToHost));
	return TG_OK;
}
