"""GPU: Tutelix (rotated latent attention, attention whose values are its keys, the gated delta rule, norms around sublayers, dense
feed-forwards, looped layers) through the C ABI against the plain statements of oracle/layers.py: every mechanism alone, prompts,
token by token, portions of many sizes, sessions used again and side by side, keys at the edges of windows, tiles and chunks, the
first tokens, long decoding, generation, the trace runner and the command line.

Tolerances are norm-relative per row: in fp32 the two sides differ by summation order, in bf16 by the rounding of the products."""
import json
import os
import subprocess

import numpy as np
import pytest

import net_models as nm
from conftest import normrel
from oracle import layers
from test_gpu_layers import F32_TOL, TOL, folder, follow, ids_of, rows_close  # noqa: F401 (folder: a fixture)

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

# heads, dim, rot_dim, vdim, q_rank, kv_rank, window, scale
LATENT = {"odd": (5, 24, 10, 36, 50, 40, 19, 0.2), "one": (1, 1, 2, 1, 1, 1, 3, 2.0), "window_1": (3, 32, 8, 20, 30, 33, 1, 0.3),
          "many_heads": (33, 32, 16, 16, 64, 70, 64, 0.2), "large": (2, 160, 96, 256, 300, 96, 65, 0.05), "rank": (4, 100, 64, 32, 40, 600, 90, 0.08),
          "square": (8, 64, 64, 64, 128, 128, 63, 0.1), "typical": (4, 128, 64, 128, 192, 320, 1000, 0.07), "negative": (2, 32, 32, 32, 48, 48, 31, -0.3)}
# heads, kv_heads, dim, rot_dims, window, scale
KEYS = {"odd": (6, 2, 20, 12, 33, 0.3), "pair": (2, 1, 2, 2, 7, 1.0), "own_keys": (5, 5, 36, 36, 50, 0.2), "one_key_head": (33, 1, 48, 16, 64, 0.15),
        "wide": (4, 2, 256, 128, 40, 0.06), "mid": (8, 4, 160, 34, 1, 0.1), "full_rot": (4, 2, 128, 128, 65, 0.1), "long": (3, 3, 64, 32, 5000, 0.15), "groups": (16, 8, 32, 2, 32, 0.2)}
# heads, kv_heads, dim, vdim, taps
DELTA = {"odd": (6, 3, 20, 12, 4), "one": (1, 1, 1, 1, 1), "slabs": (2, 2, 100, 130, 2), "wide": (2, 1, 250, 33, 3), "square": (4, 4, 64, 64, 4), "tall": (3, 1, 40, 300, 9),
         "v_mid": (2, 2, 48, 200, 70), "typical": (4, 2, 128, 128, 4), "tiles": (1, 1, 33, 16, 6)}


def check_layer(tg, cfg, path, om, dtype, n, block=1, tol=None):
    """What a layer adds to the residual stream, from a prompt and token by token; other layers' outputs do not exist."""
    ids = ids_of(cfg, n)
    taps = []
    om.step(om.state(), ids, taps)
    x0 = om.embed(ids)
    want = taps[0] - x0
    model = tg.Transformer.from_dir(path, dtype)
    s = model.open_session(n)
    s.forward(ids)
    tol = tol or TOL[dtype]
    rows_close(s.tap(0, rows=n), x0, 1e-6, "embedding")
    rows_close(s.tap(block, rows=n) - x0, want, tol, "prompt")
    s.reset()
    got = []
    for i, t in enumerate(ids):
        s.forward([t])
        got.append(s.tap(block)[0] - x0[i])
    rows_close(np.array(got), want, tol, "token by token")


def one_layer(mixer, mlp=None, width=84):
    return nm.tutelix(width, 97, [nm.layer(mixer, mlp)])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", LATENT)
def test_rotated_latent_attention_alone(tg, folder, name, dtype):
    cfg = one_layer(nm.rot_latent(*LATENT[name]))
    path, om = folder(("t_latent", name), cfg, seed=12, gain=1.5)
    check_layer(tg, cfg, path, om, dtype, 150, tol=None if dtype == "float32" else 4e-2)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", KEYS)
def test_attention_on_its_keys_alone(tg, folder, name, dtype):
    cfg = one_layer(nm.key_values(*KEYS[name]))
    path, om = folder(("t_keys", name), cfg, seed=13, gain=1.5)
    check_layer(tg, cfg, path, om, dtype, 150, tol=None if dtype == "float32" else 4e-2)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", DELTA)
def test_gated_delta_rule_alone(tg, folder, name, dtype):
    cfg = one_layer(nm.delta(*DELTA[name]))
    path, om = folder(("t_delta", name), cfg, seed=14, rank=23 if name == "slabs" else 7, gate_rank=70 if name == "square" else 5)
    # (bf16: a unit vector of one element is a sign, which can fall differently)
    check_layer(tg, cfg, path, om, dtype, 150, tol=None if dtype == "float32" else (2.5 if name == "one" else 4e-2))


@pytest.mark.parametrize("decay", [(6.0, 2.0), (-9.0, 0.5), (0.0, 8.0)])
def test_gated_delta_rule_decays(tg, folder, decay):
    """States that forget within a token, states that keep everything, and both side by side in one head."""
    cfg = one_layer(nm.delta(4, 2, 24, 16, 3), width=40)
    path, om = folder(("t_decay", decay), cfg, seed=3, decay=decay)
    check_layer(tg, cfg, path, om, "float32", 200, tol=4e-5)


def test_gated_delta_rule_on_equal_keys(tg, folder):
    """One token again and again, full step sizes, no decay: every key of a chunk is the same, the solve is at its stiffest."""
    def edit(t):
        t["l0.mix.b"] = layers.round_bf16(np.zeros_like(t["l0.mix.b"]))
        t["l0.mix.A_log"] = layers.round_bf16(np.full_like(t["l0.mix.A_log"], -12.0))
    cfg = one_layer(nm.delta(2, 1, 32, 32, 2), width=40)
    path, om = folder("t_equal", cfg, seed=4, edit=edit)
    ids = np.concatenate([np.full(90, 5), np.tile([5, 9], 30), np.full(50, 9)]).astype(np.int32)
    want = om.step(om.state(), ids)
    s = tg.Transformer.from_dir(path, "float32").open_session(200)
    rows_close(s.forward(ids, np.arange(200))[1], want, F32_TOL, "prompt")
    s.reset()
    rows_close(np.concatenate([s.forward([t])[1] for t in ids]), want, F32_TOL, "token by token")


def zero_mixer(t):
    for k in list(t):
        if k.endswith(".mix.o"):
            t[k] = np.zeros_like(t[k])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("width,ff", [(72, 40), (1, 1), (300, 1100), (2100, 64), (4200, 80)])
def test_dense_feed_forward_and_norms_alone(tg, folder, width, ff, dtype):
    """Mixers that give nothing (their norm sees zeros): widths below and above what a workgroup keeps of a row in registers."""
    cfg = one_layer(nm.delta(1, 1, 8, 8, 2), nm.dense(ff), width=width)
    path, om = folder(("t_dense", width, ff), cfg, seed=15, edit=zero_mixer)
    check_layer(tg, cfg, path, om, dtype, 40, block=2)
    ids = ids_of(cfg, 40)
    want = om.step(om.state(), ids)
    s = tg.Transformer.from_dir(path, dtype).open_session(40)
    rows_close(s.forward(ids, np.arange(40))[1], want, TOL[dtype], "logits")
    s.reset()
    rows_close(np.concatenate([s.forward([t])[1] for t in ids]), want, TOL[dtype], "logits, token by token")


# ---- whole models ------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", nm.TUTELIX)
def test_prompts_and_decoding(tg, folder, name, dtype):
    """All logits of a prompt, the residual stream behind every layer run, and the same tokens one by one."""
    cfg = nm.TUTELIX[name]
    path, om = folder(("t", name), cfg, seed=20)
    n = 140
    ids = ids_of(cfg, n, 5)
    taps = []
    want = om.step(om.state(), ids, taps)
    runs = om.runs()
    model = tg.Transformer.from_dir(path, dtype)
    assert model.architecture == "Tutelix" and model.cfg.n_vocab == cfg["vocab"] and model.cfg.n_layers == len(runs)
    s = model.open_session(n)
    # bf16: a width of 1 makes every norm a sign, and a sign can fall differently
    tol, loose = (F32_TOL, 0.0) if dtype == "float32" else (6e-2, 1.0 if name == "ones" else 0.0)
    arg, got = s.forward(ids, np.arange(n))
    rows_close(got, want, tol, "prompt logits", loose)
    if dtype == "float32":
        assert name == "ones" or arg == int(np.argmax(got[-1]))
        for r in range(len(runs)):
            rows_close(s.tap(2 * r + 2, rows=n), taps[r], F32_TOL, f"run {r}")
    s.reset()
    got = np.concatenate([s.forward([t])[1] for t in ids])
    rows_close(got, want, tol, "token by token", loose)
    if dtype == "float32":
        for r in range(len(runs)):
            rows_close(s.tap(2 * r + 2), taps[r][-1:], F32_TOL, f"run {r}, last token")


PORTIONS = {"twos": [2] * 40, "ones_and_twos": [1, 2, 1, 1, 2, 3] * 8, "edges": [63, 1, 1, 63, 2, 64, 65], "growing": [2, 3, 5, 9, 17, 33, 65, 129],
            "then_single": [100] + [1] * 40, "around_64": [64, 2, 62, 66], "behind_windows": [90, 2, 2, 41, 2, 70]}


@pytest.mark.parametrize("cut", PORTIONS)
@pytest.mark.parametrize("name", ["mixed", "flat"])
def test_portions(tg, folder, name, cut):
    cfg = nm.TUTELIX[name]
    path, om = folder(("t", name), cfg, seed=20)
    n = sum(PORTIONS[cut])
    ids = ids_of(cfg, n, 6)
    want = om.step(om.state(), ids)
    s = tg.Transformer.from_dir(path, "float32").open_session(n)
    got, at = [], 0
    for k in PORTIONS[cut]:
        got.append(s.forward(ids[at:at + k], np.arange(k))[1])
        at += k
        assert s.position == at
    rows_close(np.concatenate(got), want, F32_TOL, cut)


def test_sessions_used_again_and_side_by_side(tg, folder):
    """A reset session, a new session and sessions of unequal requests taken in turns give the same bits."""
    cfg = nm.TUTELIX["mixed"]
    path, _ = folder(("t", "mixed"), cfg, seed=20)
    model = tg.Transformer.from_dir(path, "bfloat16")
    runs = [ids_of(cfg, n, 30 + n) for n in (90, 7, 131, 1)]
    cuts = [[40, 1, 1, 48], [3, 1, 3], [2, 100, 1, 28], [1]]

    def alone(s, ids, cut):
        out, at = [], 0
        for k in cut:
            out.append(s.forward(ids[at:at + k], np.arange(k))[1])
            at += k
        return np.concatenate(out)

    fresh = [alone(model.open_session(140), r, c) for r, c in zip(runs, cuts)]
    s = model.open_session(140)
    for r, c, w in list(zip(runs, cuts, fresh)) + list(zip(runs, cuts, fresh))[::-1]:
        assert np.array_equal(alone(s, r, c), w)
        s.reset()
    sess = [model.open_session(140) for _ in runs]
    got, at = [[] for _ in runs], [0] * 4
    for step in range(4):
        for i in range(4):
            if step < len(cuts[i]):
                k = cuts[i][step]
                got[i].append(sess[i].forward(runs[i][at[i]:at[i] + k], np.arange(k))[1])
                at[i] += k
    for g, w in zip(got, fresh):
        assert np.array_equal(np.concatenate(g), w)


# ---- single keys, at the edges of windows, tiles and chunks ---------------------------------------------------------------------
def standout(om, m, q_pos, at):
    """A query token, the token whose key at position `at` scores highest with it in one of the heads, and tokens that score low
    there: the query (of 40) and head with the widest gap."""
    t, h = om.t, om.norm("l0.norm1", om.embed(np.arange(om.cfg["vocab"])))
    eps, rot, H = om.cfg["norm"]["eps"], m["rot"], m["heads"]
    if "kv_rank" in m:
        r, d = m["kv_rank"], m["dim"]
        q = (layers.rms_norm(h @ t["l0.mix.dq"].T, t["l0.mix.dq.norm"], eps) @ t["l0.mix.uq"].T).reshape(len(h), H, -1)
        kv = h @ t["l0.mix.dkv"].T
        k = (layers.rms_norm(kv[:, :r], t["l0.mix.dkv.norm"], eps) @ t["l0.mix.uk"].T).reshape(len(h), H, -1)
        qr = layers.rotate(q[:, :, d:], q_pos, rot["dims"], rot["base"], True)
        kr = layers.rotate(kv[:, r:], at, rot["dims"], rot["base"], True)
        score = np.einsum("qhd,vhd->qhv", q[:, :, :d], k) + np.einsum("qhd,vd->qhv", qr, kr)
    else:
        q = layers.rotate((h @ t["l0.mix.q"].T + t["l0.mix.q.b"]).reshape(len(h), H, -1), q_pos, rot["dims"], rot["base"], False)
        k = layers.rotate((h @ t["l0.mix.k"].T + t["l0.mix.k.b"]).reshape(len(h), m["kv_heads"], -1), at, rot["dims"], rot["base"], False)
        score = np.einsum("qhd,vhd->qhv", q, np.repeat(k, H // m["kv_heads"], 1))
    score = score[:40] * m["scale"]
    ranked = np.sort(score, -1)
    q_tok, head = np.unravel_index(np.argmax(ranked[:, :, -1] - ranked[:, :, 60]), ranked.shape[:2])
    order = np.argsort(score[q_tok, head])
    return int(q_tok), int(order[-1]), order[:60][order[:60] != q_tok]


def standout_case(om, m, n, at, seed=0):
    q_tok, key, low = standout(om, m, n - 1, at)
    plain = np.random.default_rng(seed).choice(low, n).astype(np.int32)
    plain[-1] = q_tok
    ids = plain.copy()
    ids[at] = key
    return ids, plain


WINDOWED = {"latent": lambda w: nm.rot_latent(2, 32, 16, 32, 48, 48, w, 1.0, 1e5), "keys": lambda w: nm.key_values(4, 2, 40, 24, w, 1.0, 1e5)}


@pytest.mark.parametrize("kind", WINDOWED)
@pytest.mark.parametrize("window", [1, 2, 31, 32, 33, 63, 64, 65, 130])
def test_keys_just_inside_and_just_outside_the_window(tg, folder, kind, window):
    """One key that stands out, the last that the window sees and the first that it does not: from the last place of a prompt, from
    a decoded token and from a portion of two tokens."""
    cfg = nm.tutelix(64, 211, [nm.layer(WINDOWED[kind](window))])
    path, om = folder(("t_window", kind, window), cfg, seed=41, gain=1.6)
    m, n = cfg["layers"][0]["mixer"], 200
    model = tg.Transformer.from_dir(path, "float32")
    s = model.open_session(n)
    for off in (0, 1):
        at = n - window - off
        if at == n - 1:
            continue            # a window of one sees the query's own token only
        ids, plain = standout_case(om, m, n, at)
        want, without = om.step(om.state(), ids)[-1], om.step(om.state(), plain)[-1]
        if off == 0:
            assert normrel(without, want) > 2e-2    # the key shows, 2000 times the bound
        else:
            assert np.array_equal(without, want)
        for cut in ([n], [n - 1, 1], [at + 1, n - at - 1], [n - 2, 2], [at + 1, max(n - at - 3, 0), min(2, n - at - 1)]):
            s.reset()
            p = 0
            for k in cut:
                if k:
                    got = s.forward(ids[p:p + k], [k - 1])[1]
                    p += k
            rows_close(got, want[None], F32_TOL, f"window {window}, key {at}, portions {cut}")


@pytest.mark.parametrize("kind", WINDOWED)
@pytest.mark.parametrize("at", [0, 1, 15, 16, 31, 32, 63, 64, 65, 127, 128, 191, 192, 255])
def test_one_key_that_stands_out(tg, folder, kind, at):
    """Keys at the edges of tiles under a window longer than the prompt, the first tokens among them."""
    cfg = nm.tutelix(64, 211, [nm.layer(WINDOWED[kind](300))])
    path, om = folder(("t_far", kind), cfg, seed=42, gain=1.6)
    n = 257
    ids, plain = standout_case(om, cfg["layers"][0]["mixer"], n, at)
    want, without = om.step(om.state(), ids)[-1], om.step(om.state(), plain)[-1]
    assert normrel(without, want) > 2e-2
    s = tg.Transformer.from_dir(path, "float32").open_session(n)
    for cut in ([n], [n - 1, 1], [at + 1, n - at - 1]):
        s.reset()
        p = 0
        for k in cut:
            got = s.forward(ids[p:p + k], [k - 1])[1]
            p += k
        rows_close(got, want[None], F32_TOL, f"key {at}, portions {cut}")


@pytest.mark.parametrize("at", [0, 1, 62, 63, 64, 65, 127, 128, 190, 191, 192, 195])
def test_one_write_that_stays_in_the_state(tg, folder, at):
    """The gated delta rule keeps one stand-out token over chunks: filler tokens have step sizes near zero."""
    cfg = nm.tutelix(64, 50, [nm.layer(nm.delta(2, 1, 32, 32, 3))])

    def edit(t):
        rng = np.random.default_rng(9)
        d = rng.standard_normal(64)
        t["embed"] += np.where(np.arange(50)[:, None] < 25, -3.0, 3.0) * d / np.linalg.norm(d) * 4
        t["embed"] = layers.round_bf16(t["embed"])
        t["l0.mix.b"] = layers.round_bf16(np.tile(d / np.linalg.norm(d) * 2.0, (2, 1)))
        t["l0.norm1"] *= 0
        t["l0.mix.A_log"] = layers.round_bf16(np.full(2, -6.0))
    path, om = folder("t_write", cfg, seed=43, edit=edit, decay=(-3.0, 0.3))
    n = 197
    plain = np.random.default_rng(1).integers(0, 25, n).astype(np.int32)   # fillers
    ids = plain.copy()
    ids[at] = 30
    want, without = om.step(om.state(), ids)[-1], om.step(om.state(), plain)[-1]
    assert normrel(without, want) > 2e-2
    s = tg.Transformer.from_dir(path, "float32").open_session(n)
    for cut in ([n], [n - 1, 1], [at + 1, n - at - 1], [max(at, 1), n - max(at, 1)]):
        s.reset()
        p = 0
        for k in cut:
            got = s.forward(ids[p:p + k], [k - 1])[1]
            p += k
        rows_close(got, want[None], F32_TOL, f"token {at}, portions {cut}")


def key_cache(om, h, m):
    """The oracle's cache of an attention layer from its normed inputs."""
    k = (h @ om.t["l0.mix.k"].T + om.t["l0.mix.k.b"]).reshape(len(h), m["kv_heads"], -1)
    return [(x, layers.rotate(x, p, m["rot"]["dims"], m["rot"]["base"], False)) for p, x in enumerate(k)]


@pytest.mark.parametrize("kind", WINDOWED)
@pytest.mark.parametrize("window", [700, 1100, 1500])
def test_decoding_in_long_windows(tg, folder, kind, window):
    """Windows whose decode steps take many parts (merged, folded), a key at the window's far edge, the oracle for the last query only."""
    cfg = nm.tutelix(64, 211, [nm.layer(WINDOWED[kind](window))])
    path, om = folder(("t_long", kind, window), cfg, seed=44, gain=1.6)
    n, m = 1700, cfg["layers"][0]["mixer"]
    ids, plain = standout_case(om, m, n, n - window)
    eps = cfg["norm"]["eps"]

    def last(tokens):
        h = om.norm("l0.norm1", om.embed(tokens))
        if kind == "latent":
            kv = h @ om.t["l0.mix.dkv"].T
            r = m["kv_rank"]
            cache = [(c, layers.rotate(k, p, m["rot"]["dims"], m["rot"]["base"], True))
                     for p, (c, k) in enumerate(zip(layers.rms_norm(kv[:, :r], om.t["l0.mix.dkv.norm"], eps), kv[:, r:]))]
        else:
            cache = key_cache(om, h, m)
        return om.step([cache[:-1]], tokens[-1:])

    want = last(ids)
    assert normrel(last(plain), want) > 2e-2
    for dtype in ("float32", "bfloat16"):
        s = tg.Transformer.from_dir(path, dtype).open_session(n)
        tol = F32_TOL if dtype == "float32" else 6e-2
        rows_close(s.forward(ids)[1], want, tol, "prompt")
        s.reset()
        s.forward(ids[:-1], [])
        rows_close(s.forward(ids[-1:])[1], want, tol, "decoded")


def test_long_decoding_and_several_passes(tg, folder):
    """9000 tokens: several passes of a prompt, against portions and single tokens behind them (the same bits are not asked for)."""
    cfg = nm.tutelix(64, 211, [nm.layer(nm.delta(2, 1, 32, 64, 4), nm.dense(64)), nm.layer(nm.key_values(4, 2, 32, 16, 1200, 0.3), None),
                               nm.layer(nm.rot_latent(2, 32, 16, 32, 48, 48, 5000, 0.2), nm.dense(64))], loop=(0, 2, 2))
    path, _ = folder("t_passes", cfg, seed=45, decay=(-6.0, 0.5))
    n = 9000
    ids = ids_of(cfg, n, 3)
    s = tg.Transformer.from_dir(path, "float32").open_session(n)
    want = s.forward(ids, np.arange(n - 300, n))[1]
    s.reset()
    s.forward(ids[:5001], [])
    s.forward(ids[5001:-300], [])
    rows_close(np.concatenate([s.forward([t])[1] for t in ids[-300:]]), want, 1e-4, "decoded behind 8700 tokens")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_large_products_and_tiles(tg, folder, dtype):
    """Prompts long enough for the large tiles of products and attention (places against the oracle), 32 heads."""
    cfg = nm.tutelix(190, 97, [nm.layer(nm.key_values(32, 4, 64, 32, 90, 0.2))])
    path, om = folder("t_large", cfg, seed=46)
    n = 2450
    ids = ids_of(cfg, n)
    places = [0, 1, 88, 89, 90, 91, 127, 128, 1023, 1024, 2447, 2449]
    h = om.norm("l0.norm1", om.embed(ids))
    cache = key_cache(om, h, cfg["layers"][0]["mixer"])
    want = np.concatenate([om.step([cache[:p]], ids[p:p + 1]) for p in places])
    s = tg.Transformer.from_dir(path, dtype).open_session(n)
    rows_close(s.forward(ids, places)[1], want, F32_TOL if dtype == "float32" else 5e-2, "prompt")


# ---- generation -------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("name", ["mixed", "flat"])
def test_greedy_generation(tg, folder, name):
    """tg_generate_greedy (prefill, picks and decode steps chained on the device): every pick is the oracle's, or one whose logit is
    within rounding of the oracle's best."""
    cfg = nm.TUTELIX[name]
    path, om = folder(("t", name), cfg, seed=20)
    prompt = ids_of(cfg, 30, 8)
    model = tg.Transformer.from_dir(path, "float32")
    s = model.open_session(230)
    ids, _, _ = s.greedy(prompt, 199)
    assert s.position == 229 and ids.shape == (200,)
    lg = follow(om, prompt, ids)
    gap = lg.max(-1) - lg[np.arange(200), ids]
    assert gap.max() <= 1e-4 * max(lg.std(), 1e-3), float(gap.max())
    s.reset()
    s.prefill(prompt, want_logits=False)
    s.decode_enqueue(50)
    s.decode_enqueue(149)
    assert np.array_equal(s.read_ids(200), ids)


def test_captured_steps_equal_stream_launches(tg, folder):
    """Steps replayed from captured graphs (position, windows and convolution inputs found on the device) give the picks, logits and
    residual streams of stream launches, over many replays with other work between them and across a change of the bound."""
    cfg = nm.TUTELIX["flat"]
    path, _ = folder(("t", "flat"), cfg, seed=20)
    model = tg.Transformer.from_dir(path, "bfloat16")
    prompt = ids_of(cfg, 480, 77)
    runs = {}
    for mode in (0, 1):
        tg.check(tg.lib().tg_set_graphs(mode))
        s = model.open_session(640)
        out = []
        for rep in range(3):
            s.reset()
            s.prefill(prompt[:480 - rep], want_logits=False)
            for n in (1, 7, 50, 3, 20):
                s.decode_enqueue(n)
                out.append(s.read_ids(640).tolist())
            out.append(s.tap(2 * model.cfg.n_layers)[0].tolist())
            out.append(s.decode(5)[1].tolist())
        runs[mode] = out
    tg.check(tg.lib().tg_set_graphs(-1))
    # (parts of a window are counted from its bound: sums of more parts, in another order)
    for a, b in zip(runs[0], runs[1]):
        if isinstance(a[0], int):
            assert a == b
        else:
            assert normrel(np.array(b), np.array(a)) < 2e-2


def test_sampled_generation(tg, folder):
    cfg = nm.TUTELIX["mixed"]
    path, om = folder(("t", "mixed"), cfg, seed=20)
    prompt = ids_of(cfg, 20, 9)
    s = tg.Transformer.from_dir(path, "float32").open_session(80)
    randf = np.random.default_rng(1).random(41, dtype=np.float32)
    ids, _, _ = s.generate(prompt, 40, 0.0, 0.7, randf)
    lg = follow(om, prompt, ids) / 0.7
    p = np.exp(lg - lg.max(-1, keepdims=True))
    c = np.cumsum(p / p.sum(-1, keepdims=True), -1)
    for i, t in enumerate(ids):
        lo = c[i, t - 1] if t else 0.0
        assert lo - 1e-4 <= randf[i] <= c[i, t] + 1e-4, (i, int(t))
    s.reset()
    greedy, _, _ = s.generate(prompt, 40, 1.5, 1.0, randf)
    s.reset()
    assert np.array_equal(greedy, s.greedy(prompt, 40)[0])


# ---- folders that are wrong ----------------------------------------------------------------------------------------------------
def test_folder_errors(tg, tmp_path):
    cfg = nm.tutelix(16, 20, [nm.layer(nm.rot_latent(2, 8, 4, 8, 8, 8, 5, 1.0), nm.dense(8)), nm.layer(nm.key_values(2, 1, 8, 4, 5, 1.0)),
                              nm.layer(nm.delta(2, 1, 8, 8, 2))], loop=(0, 2, 2))
    t = nm.weights(cfg, 1)
    n = [0]

    def broken(edit_cfg=None, edit_t=None):
        c, w = json.loads(json.dumps(cfg)), dict(t)
        if edit_cfg:
            edit_cfg(c)
        if edit_t:
            edit_t(w)
        n[0] += 1
        with pytest.raises(tg.TgError) as e:
            tg.Transformer.from_dir(nm.write(tmp_path / str(n[0]), c, w))
        return str(e.value)

    def mixer(i, **kw):
        return lambda c: c["layers"][i]["mixer"].update(kw)

    assert "unknown mixer" in broken(lambda c: c["layers"][0].update(type="gla"))
    assert "unknown feed-forward" in broken(lambda c: c["layers"][0]["mlp"].update(kind="moe"))
    assert "'embedding'" in broken(lambda c: c.pop("embedding"))
    assert "'vdim' must be 'dim'" in broken(mixer(1, vdim=9))
    assert "multiple of 'kv_heads'" in broken(mixer(2, kv_heads=3))
    assert "bad 'rot'" in broken(lambda c: c["layers"][1]["mixer"]["rot"].update(dims=3))
    assert "bad 'rot'" in broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=6))
    assert "'mask'" in broken(lambda c: c["layers"][0]["mixer"]["mask"].update(size=0))
    assert "no run of layers" in broken(lambda c: c["loop"].update(stop=4))
    assert "no run of layers" in broken(lambda c: c["loop"].update(start=2))
    assert "width above" in broken(lambda c: c.update(width=8000))
    assert "attention heads above" in broken(mixer(0, dim=250))
    assert "l0.norm1b" in broken(edit_t=lambda w: w.pop("l0.norm1b"))
    assert "l1.mix.k.b" in broken(edit_t=lambda w: w.pop("l1.mix.k.b"))
    assert "another shape" in broken(edit_t=lambda w: w.update({"l2.mix.k.conv": w["l2.mix.k.conv"][:, :-1]}))
    assert "another shape" in broken(edit_t=lambda w: w.update({"l2.mix.a2": w["l2.mix.a2"][:, :-1]}))
    c = json.loads(json.dumps(cfg))
    c.pop("loop")
    c["layers"][0].pop("mlp")
    model = tg.Transformer.from_dir(nm.write(tmp_path / "good", c, t))
    assert model.cfg.n_layers == 3


# ---- programs ---------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run(tg, folder, tmp_path, dtype):
    cfg = nm.TUTELIX["mixed"]
    path, om = folder(("t", "mixed"), cfg, seed=20)
    a, b = ids_of(cfg, 50, 50), ids_of(cfg, 9, 51)
    steps = [("x", a[:30], [0, 29], []), ("x", a[30:32], [], []), ("x", a[32:33], [0], []), ("x", a[33:], [16], ["x"]), ("y", b, [2, 8], ["y"]),
             ("x", a[:5], [4], ["x"])]
    text = "".join(json.dumps({"step": i, "entries": [{"id": r, "tokens": t.tolist(), "want": w}], "end": e}) + "\n"
                   for i, (r, t, w, e) in enumerate(steps))
    out = tmp_path / "out"
    out.mkdir()
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", dtype, "--out", str(out), "--max-tokens", "64"],
                       input=text, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    wa, wb = om.step(om.state(), a), om.step(om.state(), b)
    want = {0: wa[[0, 29]], 2: wa[[32]], 3: wa[[49]], 4: wb[[2, 8]], 5: wa[[4]]}
    assert sorted(os.listdir(out)) == sorted(f"{i}.f32" for i in want)
    for i, w in want.items():
        rows_close(np.fromfile(out / f"{i}.f32", "<f4").reshape(-1, cfg["vocab"]), w, F32_TOL if dtype == "float32" else 6e-2, f"step {i}")


def test_command_line(tg, folder):
    cfg = nm.TUTELIX["mixed"]
    path, _ = folder(("t", "mixed"), cfg, seed=20)
    exe = os.path.join(ROOT, "tiny-gemma_amd", "host", "gemma")
    assert os.path.exists(exe), "host/gemma is not built: run __graft_entry__.build()"
    prompt = ids_of(cfg, 12, 60)
    env = dict(os.environ, LD_LIBRARY_PATH=os.path.join(ROOT, "tiny-gemma_amd") + ":" + os.environ.get("LD_LIBRARY_PATH", ""))
    r = subprocess.run([exe, "--model_dir", path, "--dtype", "float32", "--prompt_ids", " ".join(map(str, prompt)), "--n_dec", "20"], capture_output=True,
                       text=True, env=env, timeout=100)
    assert r.returncode == 0, r.stderr
    ids = [int(x) for x in r.stdout.split("Prompt length: 12\n")[1].split("\n")[0].split()]
    s = tg.Transformer.from_dir(path, "float32").open_session(40)
    assert ids == s.greedy(prompt, 20)[0].tolist()
