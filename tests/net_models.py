"""Small random layer-list models for the tests: configurations, weights made so that faults show, model folders."""
import json
import os

import numpy as np

from oracle import layers


def gla(heads, dim, vdim, tau=16.0):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}}


def latent(heads, dim, vdim, kv_rank, scale):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale}}


def moe(experts, top, ff, scale=1.0):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "scale": scale}}


def layer(mixer, mlp=None, weights_of=None):
    l = dict(mixer, mlp=mlp)
    if weights_of is not None:
        l["weights_of"] = weights_of
    return l


def config(width, vocab, layer_list, residual_mult=0.7, eps=1e-5):
    return {"architecture": "Madevik", "width": width, "vocab": vocab, "residual_mult": residual_mult, "norm": {"eps": eps}, "layers": layer_list}


# ---- Tutelix ---------------------------------------------------------------------------------------------------------------------
def rot_latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, window, scale, base=10000.0):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                                                  "mask": {"size": window}, "rot": {"base": base, "dims": rot_dim}, "scale": scale}}


def key_values(heads, kv_heads, dim, rot_dims, window, scale, base=10000.0):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "mask": {"size": window},
                                           "rot": {"base": base, "dims": rot_dims}, "scale": scale}}


def delta(heads, kv_heads, dim, vdim, conv):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def tutelix(width, vocab, layer_list, loop=(0, 1, 1), scale=0.8, eps=1e-5):
    return {"architecture": "Tutelix", "width": width, "vocab": vocab, "embedding": {"scale": scale}, "norm": {"eps": eps},
            "layers": layer_list, "loop": {"start": loop[0], "stop": loop[1], "times": loop[2]}}


def tutelix_weights(cfg, seed, rank=7, gate_rank=5, decay=(-2.0, 1.0), gain=1.0):
    """decay: mean and spread of the decay projection's bias (large: states forget); gain: of the query and key projections."""
    rng = np.random.default_rng(seed)
    D, V = cfg["width"], cfg["vocab"]
    t = {}

    def put(name, shape, std=None, mean=0.0):
        std = (shape[-1] ** -0.5) if std is None else std
        t[name] = layers.round_bf16(rng.standard_normal(shape) * std + mean)

    put("embed", (V, D), 1.0)
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], f"l{i}.mix."
        H, d, v = m["heads"], m["dim"], m["vdim"]
        for name in ("norm1", "norm1b") + (("norm2", "norm2b") if l.get("mlp") is not None else ()):
            put(f"l{i}.{name}", (D,), 0.2)
        if l["type"] == "latent_attention":
            put(p + "dq", (m["q_rank"], D))
            put(p + "dq.norm", (m["q_rank"],), 0.2, 1.0)
            put(p + "uq", (H * (d + m["rot_dim"]), m["q_rank"]), gain * m["q_rank"] ** -0.5)
            put(p + "dkv", (m["kv_rank"] + m["rot_dim"], D), gain * D ** -0.5)
            put(p + "dkv.norm", (m["kv_rank"],), 0.2, 1.0)
            put(p + "uk", (H * d, m["kv_rank"]), gain * m["kv_rank"] ** -0.5)
            put(p + "uv", (H * v, m["kv_rank"]))
        elif l["type"] == "attention":
            G = m["kv_heads"]
            put(p + "q", (H * d, D), gain * D ** -0.5)
            put(p + "q.b", (H * d,), 0.3)
            put(p + "k", (G * d, D), gain * D ** -0.5)
            put(p + "k.b", (G * d,), 0.3)
        else:
            G = m["kv_heads"]
            for name, n in (("q", G * d), ("k", G * d), ("v", H * v)):
                put(p + name, (n, D))
                put(f"{p}{name}.conv", (n, m["conv"]), 0.7)
            put(p + "b", (H, D), 1.5 * D ** -0.5)
            put(p + "A_log", (H,), 0.5)
            put(p + "norm", (v,), 0.2, 1.0)
            put(p + "a1", (rank, D))
            put(p + "a2", (H * d, rank))
            put(p + "dt_bias", (H * d,), decay[1], decay[0])
            put(p + "g1", (gate_rank, D))
            put(p + "g2", (H * v, gate_rank))
        put(p + "o", (D, H * v))
        if l.get("mlp") is not None:
            ff = l["mlp"]["ff"]
            put(f"l{i}.mlp.up", (ff, D))
            put(f"l{i}.mlp.down", (D, ff))
    put("final.norm", (D,), 0.2)
    put("head", (V, D))
    return t


def weights(cfg, seed, **kw):
    """{name: float32 array holding bfloat16 values} of a configuration."""
    return (tutelix_weights if cfg["architecture"] == "Tutelix" else madevik_weights)(cfg, seed, **kw)


def madevik_weights(cfg, seed, rank=7, decay=(2.0, 1.5), gain=1.0):
    """decay: mean and spread of the decay projection's bias; gain: of the query and key projections (large: single keys
    stand out)."""
    rng = np.random.default_rng(seed)
    D, V = cfg["width"], cfg["vocab"]
    t = {}

    def put(name, shape, std=None, mean=0.0):
        std = (shape[-1] ** -0.5) if std is None else std
        t[name] = layers.round_bf16(rng.standard_normal(shape) * std + mean)

    def norm(name):
        put(name, (D,), 0.2, 1.0)
        put(name + ".b", (D,), 0.2)
        t[name + ".alpha"] = layers.round_bf16(np.float32(rng.uniform(0.5, 1.2))).reshape(())

    put("embed", (V, D), 1.0)
    for i, l in enumerate(cfg["layers"]):
        if l.get("weights_of") is not None:
            continue
        m, p = l["mixer"], f"l{i}.mix."
        H, d, v = m["heads"], m["dim"], m["vdim"]
        norm(f"l{i}.norm1")
        put(p + "q", (H * d, D), gain * D ** -0.5)
        put(p + "o", (D, H * v))
        if l["type"] == "gla":
            put(p + "k", (H * d, D), gain * D ** -0.5)
            put(p + "v", (H * v, D))
            put(p + "g", (H * v, D))
            put(p + "norm", (v,), 0.2, 1.0)
            put(p + "a1", (rank, D))
            put(p + "a2", (H * d, rank))
            put(p + "a2.b", (H * d,), decay[1], decay[0])
        else:
            r = m["kv_rank"]
            put(p + "dkv", (r, D))
            put(p + "dkv.norm", (r,), 0.2, 1.0)
            put(p + "uk", (H * d, r), gain * r ** -0.5)
            put(p + "uv", (H * v, r))
            put(p + "g", (H, D))
        if l.get("mlp") is not None:
            norm(f"l{i}.norm2")
            E, ff, q = l["mlp"]["router"]["experts"], l["mlp"]["expert"]["ff"], f"l{i}.mlp."
            for e in range(E):
                put(f"{q}e{e}.gate", (ff, D))
                put(f"{q}e{e}.up", (ff, D))
                put(f"{q}e{e}.down", (D, ff))
            put(q + "router", (E, D), 1.5 * D ** -0.5)
            put(q + "correction", (E,), 0.3)
    norm("final.norm")
    put("head", (V, D))
    return t


def write(path, cfg, tensors):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    layers.write_safetensors(os.path.join(path, "model.safetensors"), tensors)
    return str(path)


# Sizes that fill no tile of any kernel, sizes of 1, more heads than a tile of 16, heads above 128, layers without a
# feed-forward, one expert, all experts, shared weights (also of a layer without a feed-forward), either mixer first.
MODELS = {
    "ragged": config(84, 101, [layer(latent(5, 24, 36, 40, 0.3), moe(6, 2, 40, 1.7)), layer(gla(3, 20, 12, 4.0)), layer(gla(2, 33, 70), moe(9, 3, 25)),
                               layer(gla(3, 20, 12, 4.0), None, 1), layer(latent(5, 24, 36, 40, 0.3), moe(6, 2, 40, 1.7), 0)]),
    "wide": config(260, 1030, [layer(gla(4, 160, 96, 1.0), moe(5, 5, 70, 0.5)), layer(latent(18, 130, 200, 72, 0.1), moe(1, 1, 100, 3.0)),
                               layer(latent(18, 130, 200, 72, 0.1), moe(1, 1, 100, 3.0), 1)], residual_mult=1.0),
    "tiny": config(1, 3, [layer(gla(1, 1, 1, 2.0), moe(1, 1, 1)), layer(latent(1, 1, 1, 1, 1.0), moe(2, 1, 1)), layer(gla(1, 1, 1, 2.0))]),
    "flat": config(128, 512, [layer(latent(16, 64, 64, 512, 0.125)), layer(gla(8, 64, 128), moe(64, 8, 64, 2.0)), layer(latent(2, 32, 64, 64, 0.2))],
                   residual_mult=0.4, eps=1e-6),
}

# Tutelix: every mixer first, last and looped, layers without a feed-forward, a loop in the middle, loops of one layer, no loop,
# sizes of 1, heads that share keys and heads that do not, windows of 1 and windows longer than any prompt.
TUTELIX = {
    "mixed": tutelix(84, 101, [layer(rot_latent(5, 24, 10, 36, 50, 40, 19, 0.2), dense(70)), layer(delta(6, 2, 20, 12, 4), dense(33)),
                               layer(key_values(6, 3, 20, 12, 33, 0.2), None), layer(delta(2, 2, 33, 70, 2), dense(130))], loop=(1, 3, 3)),
    "wide": tutelix(260, 1030, [layer(key_values(36, 2, 130, 130, 70, 0.1, 500.0), dense(300)), layer(rot_latent(18, 130, 40, 200, 140, 72, 45, 0.08), None),
                                layer(delta(4, 1, 160, 96, 5), dense(260))], loop=(2, 3, 2), scale=1.7),
    "ones": tutelix(1, 3, [layer(delta(1, 1, 1, 1, 1), dense(1)), layer(key_values(1, 1, 2, 2, 1, 1.0), None), layer(rot_latent(1, 1, 2, 1, 1, 1, 1, 1.0), dense(1)),
                           layer(key_values(2, 1, 3, 2, 5, 1.0), dense(2))], loop=(0, 4, 1)),
    "flat": tutelix(128, 512, [layer(delta(8, 4, 64, 128, 3), dense(256)), layer(rot_latent(16, 64, 32, 64, 192, 128, 600, 0.1), dense(128)),
                               layer(key_values(8, 8, 64, 32, 100, 0.125, 1e6), dense(192))], loop=(0, 1, 4), scale=2.0, eps=1e-6),
}
