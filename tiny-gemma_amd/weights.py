"""Random-init weight files in the reference's on-disk format.

Counterpart, for synthetic checkpoints, of the reference's converter: the int8 weight-only
quantizer of py/weight_handlers.py:10-20 and the flat, header-less little-endian file that
py/gemma.py:27-77 writes and csrc/include/transformer.hpp:99-165 reads:

    wte int8[vocab][hidden] + f32[hidden] | RMSw f32[hidden]
    per layer: Q,K,V,O (int8 + f32 scales) | RMSq RMSk attn_pre attn_post | up, gate, down | mlp_pre mlp_post
    lm_head int8[hidden][vocab] + f32[vocab]        (tied: the transpose of the fp32 wte, re-quantized)

Matrices are [in][out] row-major with one fp32 scale per output column.

random_model_dir writes a random-init model folder (config.json + model.safetensors, bfloat16) of a layer-list model.
"""
import json
import os
import struct

import numpy as np


def quantize_weight(w):
    """scale = max|w| over axis 0 / 127 (fp32); q = rint(w / scale) as int8 (ties to even)."""
    w = np.asarray(w, np.float32)
    assert w.ndim >= 2, "Error, quantizing 1d dimensional weights"
    scales = (np.max(np.abs(w), axis=0, keepdims=True) / np.float32(127.0)).astype(np.float32)
    if not np.all(scales > 0):
        raise ZeroDivisionError("all-zero column")
    q = np.rint(w / scales).astype(np.int8)
    return q, scales


def dequantize(q, scales):
    return q.astype(np.float32) * scales


def layer_is_local(cfg, l):
    return (l % cfg.window_pattern) != (cfg.window_pattern - 1)


def weight_file_bytes(cfg):
    h, f, V, hd = cfg.hidden_size, cfg.intermediate_size, cfg.n_vocab, cfg.head_dim
    qo, kv = cfg.n_head * hd, cfg.n_kv * hd
    per_layer = (h * qo + 4 * qo) + 2 * (h * kv + 4 * kv) + (qo * h + 4 * h) + 2 * 4 * hd + 2 * 4 * h \
        + 2 * (h * f + 4 * f) + (f * h + 4 * h) + 2 * 4 * h
    return V * h + 4 * h + 4 * h + per_layer * cfg.n_layers + h * V + 4 * V


def random_weight_image(cfg, seed, std=0.02, norm_std=0.1):
    """Returns the file image (uint8 array) of a random-init model: N(0, std) matrices,
    N(0, norm_std) norm weights, lm_head tied to wte."""
    rng = np.random.default_rng(seed)
    h, f, V, hd = cfg.hidden_size, cfg.intermediate_size, cfg.n_vocab, cfg.head_dim
    qo, kv = cfg.n_head * hd, cfg.n_kv * hd
    out = np.empty(weight_file_bytes(cfg), np.uint8)
    pos = 0

    def put(a):
        nonlocal pos
        b = np.ascontiguousarray(a).view(np.uint8).reshape(-1)
        out[pos:pos + b.size] = b
        pos += b.size

    def normal(shape, s):
        return rng.standard_normal(shape, dtype=np.float32) * np.float32(s)

    def put_q(shape):
        q, s = quantize_weight(normal(shape, std))
        put(q)
        put(s)

    wte = normal((V, h), std)
    q, s = quantize_weight(wte)
    put(q)
    put(s)
    put(normal(h, norm_std))
    lm_q, lm_s = quantize_weight(np.ascontiguousarray(wte.T))
    del wte
    for _ in range(cfg.n_layers):
        put_q((h, qo))
        put_q((h, kv))
        put_q((h, kv))
        put_q((qo, h))
        put(normal(hd, norm_std))
        put(normal(hd, norm_std))
        put(normal(h, norm_std))
        put(normal(h, norm_std))
        put_q((h, f))
        put_q((h, f))
        put_q((f, h))
        put(normal(h, norm_std))
        put(normal(h, norm_std))
    put(lm_q)
    put(lm_s)
    assert pos == out.size
    return out


# ---- model folders (layer-list models) ---------------------------------------------------------------------------
def madevik_tensors(cfg, decay_rank):
    """[(name, shape, kind)] of a Madevik model in file order; kind: "w" matrix, "one" norm weight, "zero" bias,
    "alpha" scalar of the element-wise tanh norm, "decay" and "softplus" bias of a decay projection."""
    D, V = cfg["width"], cfg["vocab"]
    out = [("embed", (V, D), "w")]

    def norm(name):
        out.extend([(name, (D,), "one"), (name + ".b", (D,), "zero"), (name + ".alpha", (), "alpha")])

    for i, l in enumerate(cfg["layers"]):
        if l.get("weights_of") is not None:
            continue
        m, p = l["mixer"], f"l{i}.mix."
        H, d, v = m["heads"], m["dim"], m["vdim"]
        norm(f"l{i}.norm1")
        if l["type"] == "gla":
            out += [(p + "q", (H * d, D), "w"), (p + "k", (H * d, D), "w"), (p + "v", (H * v, D), "w"), (p + "g", (H * v, D), "w"),
                    (p + "o", (D, H * v), "w"), (p + "norm", (v,), "one"), (p + "a1", (decay_rank, D), "w"), (p + "a2", (H * d, decay_rank), "w"),
                    (p + "a2.b", (H * d,), "decay")]
        else:
            r = m["kv_rank"]
            out += [(p + "q", (H * d, D), "w"), (p + "dkv", (r, D), "w"), (p + "dkv.norm", (r,), "one"), (p + "uk", (H * d, r), "w"),
                    (p + "uv", (H * v, r), "w"), (p + "g", (H, D), "w"), (p + "o", (D, H * v), "w")]
        if l.get("mlp") is not None:
            norm(f"l{i}.norm2")
            E, ff, q = l["mlp"]["router"]["experts"], l["mlp"]["expert"]["ff"], f"l{i}.mlp."
            for e in range(E):
                out += [(f"{q}e{e}.gate", (ff, D), "w"), (f"{q}e{e}.up", (ff, D), "w"), (f"{q}e{e}.down", (D, ff), "w")]
            out += [(q + "router", (E, D), "w"), (q + "correction", (E,), "zero")]
    norm("final.norm")
    out.append(("head", (V, D), "w"))
    return out


def tutelix_tensors(cfg, decay_rank, gate_rank):
    """The same of a Tutelix model (norm weights stored around zero, A_log and convolutions are "zero" and "w")."""
    D, V = cfg["width"], cfg["vocab"]
    out = [("embed", (V, D), "w")]
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], f"l{i}.mix."
        H, d, v = m["heads"], m["dim"], m["vdim"]
        mlp = l.get("mlp")
        out += [(f"l{i}.{n}", (D,), "zero") for n in ("norm1", "norm1b") + (("norm2", "norm2b") if mlp else ())]
        if l["type"] == "latent_attention":
            q, r, e = m["q_rank"], m["kv_rank"], m["rot_dim"]
            out += [(p + "dq", (q, D), "w"), (p + "dq.norm", (q,), "one"), (p + "uq", (H * (d + e), q), "w"), (p + "dkv", (r + e, D), "w"),
                    (p + "dkv.norm", (r,), "one"), (p + "uk", (H * d, r), "w"), (p + "uv", (H * v, r), "w")]
        elif l["type"] == "attention":
            G = m["kv_heads"]
            out += [(p + "q", (H * d, D), "w"), (p + "q.b", (H * d,), "zero"), (p + "k", (G * d, D), "w"), (p + "k.b", (G * d,), "zero")]
        else:
            G = m["kv_heads"]
            for n, rows in (("q", G * d), ("k", G * d), ("v", H * v)):
                out += [(p + n, (rows, D), "w"), (f"{p}{n}.conv", (rows, m["conv"]), "w")]
            out += [(p + "b", (H, D), "w"), (p + "A_log", (H,), "zero"), (p + "norm", (v,), "one"), (p + "a1", (decay_rank, D), "w"),
                    (p + "a2", (H * d, decay_rank), "w"), (p + "dt_bias", (H * d,), "softplus"), (p + "g1", (gate_rank, D), "w"),
                    (p + "g2", (H * v, gate_rank), "w")]
        out.append((p + "o", (D, H * v), "w"))
        if mlp:
            out += [(f"l{i}.mlp.up", (mlp["ff"], D), "w"), (f"l{i}.mlp.down", (D, mlp["ff"]), "w")]
    return out + [("final.norm", (D,), "zero"), ("head", (V, D), "w")]


def random_model_dir(path, cfg, seed, decay_rank=16, block=1 << 22, gate_rank=None):
    """Writes config.json and model.safetensors of a random-init model (matrices N(0, 1 / inputs)) into `path`.  Matrices are
    cut at random places out of one block of normal numbers per scale: large models are written at the speed of the disk."""
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    rng = np.random.default_rng(seed)
    base = rng.standard_normal(block, dtype=np.float32)

    def bf16(a):
        u = np.ascontiguousarray(a, np.float32).view(np.uint32)
        return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)

    blocks = {}
    head, off = {}, 0
    tensors = tutelix_tensors(cfg, decay_rank, gate_rank or decay_rank) if cfg["architecture"] == "Tutelix" else madevik_tensors(cfg, decay_rank)
    for name, shape, _ in tensors:
        n = 2 * int(np.prod(shape, dtype=np.int64))
        head[name] = {"dtype": "BF16", "shape": list(shape), "data_offsets": [off, off + n]}
        off += n
    text = json.dumps(head).encode()
    text += b" " * (-len(text) % 8)
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(text)) + text)
        for _, shape, kind in tensors:
            n = int(np.prod(shape, dtype=np.int64))
            if kind == "w":
                std = float(shape[-1]) ** -0.5
                if std not in blocks:
                    blocks[std] = bf16(base * np.float32(std))
                b = blocks[std]
                while n > 0:
                    k = min(n, block // 2)
                    at = int(rng.integers(0, block - k + 1))
                    f.write(b[at:at + k].tobytes())
                    n -= k
            else:
                a = {"one": 1.0, "zero": 0.0, "alpha": 0.7, "decay": 3.0, "softplus": -3.0}[kind] * np.ones(n, np.float32)
                if kind in ("one", "zero"):
                    a += rng.standard_normal(n, dtype=np.float32) * np.float32(0.1)
                f.write(bf16(a).tobytes())
