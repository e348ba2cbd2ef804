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


def weights(cfg, seed, rank=7, decay=(2.0, 1.5), gain=1.0):
    """{name: float32 array holding bfloat16 values}.  decay: mean and spread of the decay projection's bias; gain: of the
    query and key projections (large: single keys stand out)."""
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
