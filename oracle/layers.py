"""Plain statements of the mechanisms of the layer-list models (decoder-only models whose config.json lists their layers
one by one), one function per mechanism, in numpy and in double precision: test infrastructure, shares nothing with the
product.  Everything is written for reading, token by token, from the equations.

Shapes: n tokens, width D, H heads.  Weights are [out, in].
"""
import json
import math
import os
import struct

import numpy as np

F = np.float64


# ---- storage -----------------------------------------------------------------------------------
def to_bf16_bits(a):
    """float32 -> bfloat16 bit patterns, round to nearest even."""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def from_bf16_bits(b):
    return (np.asarray(b, np.uint16).astype(np.uint32) << 16).view(np.float32)


def round_bf16(a):
    return from_bf16_bits(to_bf16_bits(a))


def write_safetensors(path, tensors):
    """{name: float array} as bfloat16, in the given order."""
    head, blobs, off = {}, [], 0
    for name, a in tensors.items():
        raw = to_bf16_bits(np.asarray(a, np.float32)).tobytes()
        head[name] = {"dtype": "BF16", "shape": list(np.shape(a)), "data_offsets": [off, off + len(raw)]}
        blobs.append(raw)
        off += len(raw)
    h = json.dumps(head).encode()
    h += b" " * (-len(h) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h)
        for b in blobs:
            f.write(b)


def read_safetensors(path):
    """{name: float32 array} of a file of bfloat16 / float32 / int32 tensors."""
    with open(path, "rb") as f:
        n = struct.unpack("<Q", f.read(8))[0]
        head = json.loads(f.read(n))
        data = f.read()
    out = {}
    for name, t in head.items():
        if name == "__metadata__":
            continue
        raw = data[t["data_offsets"][0]:t["data_offsets"][1]]
        if t["dtype"] == "BF16":
            a = from_bf16_bits(np.frombuffer(raw, np.uint16))
        elif t["dtype"] == "F32":
            a = np.frombuffer(raw, np.float32)
        else:
            a = np.frombuffer(raw, np.int32)
        out[name] = a.reshape(t["shape"])
    return out


# ---- elementary functions ------------------------------------------------------------------------
def sigmoid(z):
    z = np.asarray(z, F)
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def log_sigmoid(z):
    z = np.asarray(z, F)
    return np.minimum(z, 0.0) - np.log1p(np.exp(-np.abs(z)))


def silu(z):
    return z * sigmoid(z)


# ---- norms -----------------------------------------------------------------------------------------
def dynamic_tanh(x, alpha, w, b):
    """tanh(alpha x) w + b, element by element."""
    return np.tanh(F(alpha) * x) * w + b


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def centred_rms_norm(x, w, eps):
    """The weight is stored as its distance from one."""
    return rms_norm(x, 1.0 + w, eps)


# ---- latent attention -------------------------------------------------------------------------------
def latent_attention(h, cache, w, heads, dim, vdim, scale, eps):
    """h [n, D]; cache: list of latent rows seen so far (extended in place); w: dict q, dkv, dkv_norm, uk, uv, g, o.

    c = rms(Wdkv h), k_head = Wuk c, v_head = Wuv c; token i sees every row up to its own; softmax of scale * q.k; the
    head's value sum times sigmoid(Wg h)_head."""
    out = np.zeros((h.shape[0], w["o"].shape[0]), F)
    for i in range(h.shape[0]):
        cache.append(rms_norm(w["dkv"] @ h[i], w["dkv_norm"], eps))
        c = np.stack(cache)
        q = (w["q"] @ h[i]).reshape(heads, dim)
        gate = sigmoid(w["g"] @ h[i])
        heads_out = []
        for a in range(heads):
            k = c @ w["uk"][a * dim:(a + 1) * dim].T
            v = c @ w["uv"][a * vdim:(a + 1) * vdim].T
            s = (k @ q[a]) * scale
            p = np.exp(s - s.max())
            heads_out.append(gate[a] * ((p / p.sum()) @ v))
        out[i] = w["o"] @ np.concatenate(heads_out)
    return out


# ---- gated linear attention ---------------------------------------------------------------------------
def gla(h, state, w, heads, dim, vdim, tau, eps):
    """h [n, D]; state [H, dim, vdim], updated in place; w: dict q, k, v, g, o, norm, a1, a2, a2_b.

    Per head S <- diag(alpha) S + k v^T with alpha = sigmoid(z)^(1/tau) per key channel, o = S^T q."""
    out = np.zeros((h.shape[0], w["o"].shape[0]), F)
    for t in range(h.shape[0]):
        x = h[t]
        q = (w["q"] @ x).reshape(heads, dim) * dim ** -0.5
        k = (w["k"] @ x).reshape(heads, dim)
        v = (w["v"] @ x).reshape(heads, vdim)
        z = w["a2"] @ (w["a1"] @ x) + w["a2_b"]
        alpha = np.exp(log_sigmoid(z) / tau).reshape(heads, dim)
        heads_out = []
        for a in range(heads):
            state[a] = alpha[a][:, None] * state[a] + np.outer(k[a], v[a])
            heads_out.append(rms_norm(state[a].T @ q[a], w["norm"], eps))
        out[t] = w["o"] @ (np.concatenate(heads_out) * silu(w["g"] @ x))
    return out


# ---- rotary positions ---------------------------------------------------------------------------------------
def rotate(x, pos, dims, base, interleaved):
    """x [..., size]: its first `dims` elements turned by pos * base^(-2i / dims), i = 0 .. dims / 2 - 1; pairs (2i, 2i + 1)
    or (i, i + dims / 2)."""
    out = np.array(x, F)
    for i in range(dims // 2):
        a, b = (2 * i, 2 * i + 1) if interleaved else (i, i + dims // 2)
        t = pos * F(base) ** (-2.0 * i / dims)
        out[..., a] = x[..., a] * np.cos(t) - x[..., b] * np.sin(t)
        out[..., b] = x[..., b] * np.cos(t) + x[..., a] * np.sin(t)
    return out


# ---- latent attention with a latent query, a rotated key part shared by the heads, and a window ----------------------
def softmax_sum(scores, values):
    p = np.exp(scores - scores.max())
    return (p / p.sum()) @ values


def rotated_latent_attention(h, cache, w, heads, dim, rot_dim, vdim, scale, window, dims, base, eps):
    """h [n, D]; cache: list of (latent, rotated key part), one per token seen (extended in place).

    q = Wuq rms(Wdq h), per head [dim | rot_dim]; Wdkv h = [latent before its norm | key part]; a head's score with token j is
    (q . Wuk c_j + rot(q') . rot(k'_j)) * scale over the last `window` tokens, its values are Wuv c_j."""
    out = np.zeros((h.shape[0], w["o"].shape[0]), F)
    rank = w["uk"].shape[1]
    for t in range(h.shape[0]):
        pos = len(cache)
        kv = w["dkv"] @ h[t]
        cache.append((rms_norm(kv[:rank], w["dkv_norm"], eps), rotate(kv[rank:], pos, dims, base, True)))
        lo = max(0, pos - window + 1)
        c = np.stack([r[0] for r in cache[lo:]])
        kr = np.stack([r[1] for r in cache[lo:]])
        q = (w["uq"] @ rms_norm(w["dq"] @ h[t], w["dq_norm"], eps)).reshape(heads, dim + rot_dim)
        qr = rotate(q[:, dim:], pos, dims, base, True)
        heads_out = []
        for a in range(heads):
            k = c @ w["uk"][a * dim:(a + 1) * dim].T
            v = c @ w["uv"][a * vdim:(a + 1) * vdim].T
            heads_out.append(softmax_sum((k @ q[a, :dim] + kr @ qr[a]) * scale, v))
        out[t] = w["o"] @ np.concatenate(heads_out)
    return out


# ---- attention whose values are its keys --------------------------------------------------------------------------
def key_value_attention(h, cache, w, heads, kv_heads, dim, scale, window, dims, base):
    """h [n, D]; cache: list of (keys [kv_heads, dim] as projected, the same rotated), extended in place.  Query head a uses key head
    a // (heads / kv_heads); scores on rotated queries and keys over the last `window` tokens; the values are the keys as
    projected."""
    out = np.zeros((h.shape[0], w["o"].shape[0]), F)
    for t in range(h.shape[0]):
        pos = len(cache)
        key = (w["k"] @ h[t] + w["k_b"]).reshape(kv_heads, dim)
        cache.append((key, rotate(key, pos, dims, base, False)))
        q = rotate((w["q"] @ h[t] + w["q_b"]).reshape(heads, dim), pos, dims, base, False)
        lo = max(0, pos - window + 1)
        v = np.stack([c[0] for c in cache[lo:]])
        k = np.stack([c[1] for c in cache[lo:]])
        heads_out = []
        for a in range(heads):
            g = a // (heads // kv_heads)
            heads_out.append(softmax_sum(k[:, g] @ q[a] * scale, v[:, g]))
        out[t] = w["o"] @ np.concatenate(heads_out)
    return out


# ---- gated delta rule with a decay per key channel ------------------------------------------------------------------
def short_conv(x, past, taps):
    """x [channels]: the newest input; past: list of the inputs before it (extended in place); taps [channels, n], the last
    column meets x."""
    past.append(np.array(x, F))
    n = taps.shape[1]
    out = np.zeros_like(past[-1])
    for i in range(n):
        at = len(past) - n + i
        if at >= 0:
            out += taps[:, i] * past[at]
    return out


def softplus(z):
    return -log_sigmoid(-np.asarray(z, F))


def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def delta_state(heads, dim, vdim):
    return {"S": np.zeros((heads, dim, vdim), F), "q": [], "k": [], "v": []}


def channel_delta(h, state, w, heads, kv_heads, dim, vdim, eps):
    """h [n, D]; state: delta_state(), updated in place.

    Per head S <- diag(g) S, u = beta (v - S^T k), S <- S + k u^T, o = S^T q."""
    out = np.zeros((h.shape[0], w["o"].shape[0]), F)
    for t in range(h.shape[0]):
        x = h[t]
        q, k, v = (silu(short_conv(w[n] @ x, state[n], w[n + "_conv"])) for n in ("q", "k", "v"))
        q = unit(q.reshape(kv_heads, dim)) * dim ** -0.5
        k = unit(k.reshape(kv_heads, dim))
        v = v.reshape(heads, vdim)
        beta = sigmoid(w["b"] @ x)
        z = (w["a2"] @ (w["a1"] @ x) + w["dt_bias"]).reshape(heads, dim)
        g = np.exp(-np.exp(w["A_log"])[:, None] * softplus(z))
        heads_out = []
        for a in range(heads):
            S, c = state["S"][a], a // (heads // kv_heads)
            S *= g[a][:, None]
            u = beta[a] * (v[a] - S.T @ k[c])
            S += np.outer(k[c], u)
            heads_out.append(rms_norm(S.T @ q[c], w["norm"], eps))
        out[t] = w["o"] @ (np.concatenate(heads_out) * sigmoid(w["g2"] @ (w["g1"] @ x)))
    return out


# ---- dense feed-forward ---------------------------------------------------------------------------------------------
_erf = np.vectorize(math.erf, otypes=[F])


def gelu(z):
    z = np.asarray(z, F)
    return 0.5 * z * (1.0 + _erf(z / np.sqrt(F(2.0))))


def dense(h, up, down):
    return gelu(h @ up.T) @ down.T


# ---- experts ---------------------------------------------------------------------------------------------
def route(scores, correction, top, scale):
    """scores [E] after the sigmoid -> (chosen experts, their weights): chosen by scores + correction (the lower index
    wins a tie), weighted by the scores themselves, normalised over the chosen, times scale."""
    order = sorted(range(len(scores)), key=lambda e: (-(scores[e] + correction[e]), e))[:top]
    s = np.array([scores[e] for e in order], F)
    return order, s / (s.sum() + 1e-20) * scale


def mixture(h, w, experts, top, scale):
    """h [n, D]; w: dict router, correction, gate/up/down: lists per expert."""
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        chosen, weights = route(sigmoid(w["router"] @ h[t]), w["correction"], top, scale)
        for e, g in zip(chosen, weights):
            out[t] += g * (w["down"][e] @ (silu(w["gate"][e] @ h[t]) * (w["up"][e] @ h[t])))
    return out


# ---- the model ---------------------------------------------------------------------------------------------
class LayerModel:
    """A model from its config (dict) and tensors ({name: array}); state() makes one sequence's caches and states."""

    def __init__(self, cfg, tensors):
        self.cfg = cfg
        self.t = {k: np.asarray(v, F) for k, v in tensors.items()}

    @classmethod
    def from_dir(cls, path):
        with open(os.path.join(path, "config.json")) as f:
            cfg = json.load(f)
        cls = DESIGNS[cfg["architecture"]]
        return cls(cfg, read_safetensors(os.path.join(path, "model.safetensors")))

    def state(self):
        s = []
        for l in self.cfg["layers"]:
            m = l["mixer"]
            s.append([] if l["type"] == "latent_attention" else np.zeros((m["heads"], m["dim"], m["vdim"]), F))
        return s

    def norm(self, name, x):
        return dynamic_tanh(x, self.t[name + ".alpha"], self.t[name], self.t[name + ".b"])

    def mixer(self, i, h, state):
        l = self.cfg["layers"][i]
        m, t, p = l["mixer"], self.t, f"l{l.get('weights_of', i)}.mix."
        eps = self.cfg["norm"]["eps"]
        if l["type"] == "latent_attention":
            w = {k: t[p + k] for k in ("q", "dkv", "uk", "uv", "g", "o")}
            w["dkv_norm"] = t[p + "dkv.norm"]
            return latent_attention(h, state, w, m["heads"], m["dim"], m["vdim"], m["scale"], eps)
        w = {k: t[p + k] for k in ("q", "k", "v", "g", "o", "norm", "a1", "a2")}
        w["a2_b"] = t[p + "a2.b"]
        return gla(h, state, w, m["heads"], m["dim"], m["vdim"], m["tau"], eps)

    def feed_forward(self, i, h):
        l = self.cfg["layers"][i]
        r, t, p = l["mlp"]["router"], self.t, f"l{l.get('weights_of', i)}.mlp."
        w = {"router": t[p + "router"], "correction": t[p + "correction"]}
        for k in ("gate", "up", "down"):
            w[k] = [t[f"{p}e{e}.{k}"] for e in range(r["experts"])]
        return mixture(h, w, r["experts"], r["top"], r["scale"])

    def step(self, state, tokens, taps=None):
        """Runs `tokens` from `state`; logits [n, vocab].  taps: list that receives the residual stream after every layer."""
        m = self.cfg["residual_mult"]
        x = self.t["embed"][np.asarray(tokens, np.int64)].copy()
        for i, l in enumerate(self.cfg["layers"]):
            p = f"l{l.get('weights_of', i)}."
            x = x + m * self.mixer(i, self.norm(p + "norm1", x), state[i])
            if l.get("mlp") is not None:
                x = x + m * self.feed_forward(i, self.norm(p + "norm2", x))
            if taps is not None:
                taps.append(x.copy())
        return self.norm("final.norm", x) @ self.t["head"].T

    def greedy(self, prompt, n):
        """The prompt's greedy continuation: n + 1 ids and, for each, the gap between the two best logits."""
        state = self.state()
        ids, gaps = [], []
        logits = self.step(state, prompt)[-1]
        while True:
            order = np.argsort(-logits, kind="stable")
            ids.append(int(order[0]))
            gaps.append(float(logits[order[0]] - logits[order[1]]))
            if len(ids) == n + 1:
                return ids, gaps
            logits = self.step(state, [ids[-1]])[-1]



class TutelixModel(LayerModel):
    """Norms before and after each sublayer, windowed attention of two kinds, the gated delta rule, dense feed-forwards, a run
    of layers that is passed several times with its own caches and states each time."""

    def runs(self):
        """The layer of every layer run."""
        n, loop = len(self.cfg["layers"]), self.cfg.get("loop")
        if not loop:
            return list(range(n))
        a, b = loop["start"], loop["stop"]
        return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))

    def state(self):
        s = []
        for i in self.runs():
            l = self.cfg["layers"][i]
            m = l["mixer"]
            s.append(delta_state(m["heads"], m["dim"], m["vdim"]) if l["type"] == "channel_delta" else [])
        return s

    def norm(self, name, x):
        return centred_rms_norm(x, self.t[name], self.cfg["norm"]["eps"])

    def mixer(self, i, h, state):
        l = self.cfg["layers"][i]
        m, t, p, eps = l["mixer"], self.t, f"l{i}.mix.", self.cfg["norm"]["eps"]

        def pick(*names):
            return {n.replace(".b", "_b").replace(".", "_"): t[p + n] for n in names}

        if l["type"] == "latent_attention":
            return rotated_latent_attention(h, state, pick("dq", "dq.norm", "uq", "dkv", "dkv.norm", "uk", "uv", "o"), m["heads"], m["dim"], m["rot_dim"],
                                            m["vdim"], m["scale"], m["mask"]["size"], m["rot"]["dims"], m["rot"]["base"], eps)
        if l["type"] == "attention":
            return key_value_attention(h, state, pick("q", "q.b", "k", "k.b", "o"), m["heads"], m["kv_heads"], m["dim"], m["scale"],
                                       m["mask"]["size"], m["rot"]["dims"], m["rot"]["base"])
        w = pick("q", "q.conv", "k", "k.conv", "v", "v.conv", "b", "a1", "a2", "dt_bias", "A_log", "norm", "g1", "g2", "o")
        return channel_delta(h, state, w, m["heads"], m["kv_heads"], m["dim"], m["vdim"], eps)

    def embed(self, tokens):
        return self.t["embed"][np.asarray(tokens, np.int64)] * self.cfg["embedding"]["scale"]

    def feed_forward(self, i, h):
        return dense(h, self.t[f"l{i}.mlp.up"], self.t[f"l{i}.mlp.down"])

    def step(self, state, tokens, taps=None):
        x = self.embed(tokens)
        for r, i in enumerate(self.runs()):
            p = f"l{i}."
            x = x + self.norm(p + "norm1b", self.mixer(i, self.norm(p + "norm1", x), state[r]))
            if self.cfg["layers"][i].get("mlp") is not None:
                x = x + self.norm(p + "norm2b", self.feed_forward(i, self.norm(p + "norm2", x)))
            if taps is not None:
                taps.append(x.copy())
        return self.norm("final.norm", x) @ self.t["head"].T


DESIGNS = {"Madevik": LayerModel, "Tutelix": TutelixModel}


def model_of(cfg, tensors):
    return DESIGNS[cfg["architecture"]](cfg, tensors)
