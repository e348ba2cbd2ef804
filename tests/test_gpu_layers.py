"""GPU: layer-list models (gated linear attention, latent attention, element-wise tanh norms, mixtures of experts) through
the C ABI against the plain statements of oracle/layers.py: every mechanism alone, whole prompts, token by token, portions
of many sizes, sessions used again and side by side, keys far away, long decoding, generation and the trace runner.

Tolerances are norm-relative per row.  In fp32 the two sides differ by summation order; in bf16 by the rounding of weights'
products (the oracle computes in double precision on the same bfloat16 weights), and where a mixture of experts is involved a
close choice may fall differently on a few rows."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import net_models as nm
from conftest import normrel
from oracle import layers

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F32_TOL, BF16_TOL = 1e-5, 3e-2
TOL = {"float32": F32_TOL, "bfloat16": BF16_TOL}


@pytest.fixture(scope="module")
def folder(tmp_path_factory):
    """(path, oracle model) of a configuration, written once."""
    cache = {}

    def make(key, cfg, seed=1, edit=None, **kw):
        if key not in cache:
            t = nm.weights(cfg, seed, **kw)
            if edit:
                edit(t)
            cache[key] = (nm.write(tmp_path_factory.mktemp("net") / "m", cfg, t), layers.model_of(cfg, t))
        return cache[key]

    return make


def rows_close(got, want, tol, what, loose_rows=0.0):
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    assert got.shape == want.shape and np.isfinite(got).all()
    scale = np.sqrt((want ** 2).sum(-1)).mean()
    err = np.sqrt(((got - want) ** 2).sum(-1)) / max(scale, 1e-30)
    over = int((err > tol).sum())
    print(f"{what}: worst row {err.max():.2e}, median {np.median(err):.2e} (bound {tol:.0e}, {over} of {err.size} over)", flush=True)
    assert over <= loose_rows * err.size, (what, float(err.max()))


def ids_of(cfg, n, seed=0):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).astype(np.int32)


# ---- one mechanism at a time: models of a single layer, the others' outputs made zero -------------------------------------
GLA_SIZES = {"odd": (3, 20, 12, 4.0), "one": (1, 1, 1, 1.0), "slabs": (2, 100, 130, 16.0), "wide": (2, 257, 33, 2.0), "square": (4, 64, 64, 8.0), "tall": (1, 40, 300, 4.0),
             "v_mid": (2, 48, 200, 8.0)}
LATENT_SIZES = {"odd": (5, 24, 36, 40, 0.3), "one": (1, 1, 1, 1, 2.0), "many_heads": (33, 32, 16, 70, 0.2), "large": (2, 200, 256, 96, 0.1),
                "v_small": (4, 128, 32, 600, 0.08), "square": (8, 64, 64, 128, 0.125), "v_wide": (3, 40, 100, 50, 0.2),
                "both_128": (2, 100, 128, 64, 0.15), "q_wide": (2, 160, 96, 64, 0.1), "negative": (2, 32, 32, 48, -0.3)}
MOE_SIZES = {"odd": (6, 2, 40, 1.7), "one": (1, 1, 1, 2.0), "all": (7, 7, 33, 0.3), "many": (130, 6, 20, 2.5), "top1": (16, 1, 96, 1.0), "crowd": (300, 5, 16, 1.0)}


def mixer_case(folder, kind, name, width=84):
    if kind == "gla":
        cfg = nm.config(width, 97, [nm.layer(nm.gla(*GLA_SIZES[name]))])
        return cfg, *folder(("gla", name), cfg, seed=11, gain=1.5, rank=23 if name == "slabs" else 7)
    cfg = nm.config(width, 97, [nm.layer(nm.latent(*LATENT_SIZES[name]))])
    return cfg, *folder(("latent", name), cfg, seed=12, gain=2.0)


def check_block(tg, cfg, path, om, dtype, n, block=1, loose_rows=0.0, tol=None):
    """Residual stream behind the layer, from a prompt and token by token."""
    ids = ids_of(cfg, n)
    taps = []
    om.step(om.state(), ids, taps)
    x0 = om.t["embed"][ids]
    want = taps[0] - x0
    model = tg.Transformer.from_dir(path, dtype)
    s = model.open_session(n)
    s.forward(ids)
    tol = tol or TOL[dtype]
    assert np.array_equal(s.tap(0, rows=n) if n > 1 else s.tap(0), x0.astype(np.float32))
    rows_close(s.tap(block, rows=n) - x0, want, tol, "prompt", loose_rows)
    s.reset()
    got = []
    for t in ids:
        s.forward([t])
        got.append(s.tap(block)[0] - om.t["embed"][t])
    rows_close(np.array(got), want, tol, "token by token", loose_rows)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", GLA_SIZES)
def test_gated_linear_attention_alone(tg, folder, name, dtype):
    cfg, path, om = mixer_case(folder, "gla", name)
    check_block(tg, cfg, path, om, dtype, 150)


@pytest.mark.parametrize("decay,tau", [((-6.0, 2.0), 0.5), ((8.0, 0.5), 16.0), ((0.0, 8.0), 1.0)])
def test_gated_linear_attention_decays(tg, folder, decay, tau):
    """States that forget within a token, states that keep everything, and both side by side in one head: the chunked
    form must neither overflow nor lose the near tokens."""
    cfg = nm.config(40, 97, [nm.layer(nm.gla(2, 24, 16, tau))])
    path, om = folder(("decay", decay), cfg, seed=3, decay=decay)
    check_block(tg, cfg, path, om, "float32", 200, tol=4e-5)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", LATENT_SIZES)
def test_latent_attention_alone(tg, folder, name, dtype):
    cfg, path, om = mixer_case(folder, "latent", name)
    check_block(tg, cfg, path, om, dtype, 150)


def zero_mixer(t):
    for k in list(t):
        if k.endswith(".mix.o"):
            t[k] = np.zeros_like(t[k])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", MOE_SIZES)
def test_experts_alone(tg, folder, name, dtype):
    cfg = nm.config(72, 97, [nm.layer(nm.gla(1, 8, 8), nm.moe(*MOE_SIZES[name]))])
    path, om = folder(("moe", name), cfg, seed=13, edit=zero_mixer)
    check_block(tg, cfg, path, om, dtype, 150, block=2, loose_rows=0.0 if dtype == "float32" else 0.08)


def test_many_rows_per_expert(tg, folder):
    """Enough tokens for the 128-row tiles of the grouped product, with experts that get none of them."""
    def edit(t):
        zero_mixer(t)
        t["l0.mlp.correction"] = layers.round_bf16(np.array([0, 0, -9.0, 0, -9.0], np.float32))
    cfg = nm.config(72, 97, [nm.layer(nm.gla(1, 8, 8), nm.moe(5, 2, 40, 1.5))])
    path, om = folder("moe_rows", cfg, seed=14, edit=edit)
    check_block(tg, cfg, path, om, "float32", 700, block=2)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n", [700, 2450])
def test_large_products(tg, folder, dtype, n):
    """Prompts long enough for the 64- and 128-row tiles of the plain products (3072 columns), with an odd number of stages."""
    cfg = nm.config(190, 97, [nm.layer(nm.gla(8, 64, 128, 8.0))])
    path, om = folder("large", cfg, seed=16)
    ids = ids_of(cfg, n)
    taps = []
    om.step(om.state(), ids, taps)
    s = tg.Transformer.from_dir(path, dtype).open_session(n)
    want = np.arange(0, n, 7)
    got = s.forward(ids, want)[1]
    rows_close(got, om.norm("final.norm", taps[0][want]) @ om.t["head"].T, TOL[dtype], f"{n} tokens")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_many_heads_and_a_long_prompt(tg, folder, dtype):
    """64 heads and 1030 tokens: the 128-query tiles of the attention kernel; places at their edges against the oracle."""
    cfg = nm.config(64, 97, [nm.layer(nm.latent(64, 32, 32, 64, 0.4))])
    path, om = folder("many_heads", cfg, seed=17, gain=1.5)
    n = 1030
    ids = ids_of(cfg, n)
    c = om.norm("l0.norm1", om.t["embed"][ids]) @ om.t["l0.mix.dkv"].T
    cache = list(layers.rms_norm(c, om.t["l0.mix.dkv.norm"], cfg["norm"]["eps"]))
    places = [0, 15, 16, 63, 64, 127, 128, 129, 511, 512, 1023, 1024, 1029]
    want = np.concatenate([om.step([cache[:p]], ids[p:p + 1]) for p in places])
    s = tg.Transformer.from_dir(path, dtype).open_session(n)
    rows_close(s.forward(ids, places)[1], want, TOL[dtype], "whole")
    s.reset()
    s.forward(ids[:100], [])
    rows_close(s.forward(ids[100:], [p - 100 for p in places if p >= 100])[1], want[[p >= 100 for p in places]], TOL[dtype], "behind 100 tokens")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_wide_decode_products(tg, folder, dtype):
    """A vocabulary of thousands of tiles (a wave per tile in the head) and a layer whose products take two tiles per
    workgroup, with an odd one left over."""
    cfg = nm.config(32, 33001, [nm.layer(nm.gla(2, 8, 8)), nm.layer(nm.gla(16, 96, 128))])
    path, om = folder("wide_decode", cfg, seed=18)
    ids = ids_of(cfg, 24)
    want = om.step(om.state(), ids)
    s = tg.Transformer.from_dir(path, dtype).open_session(64)
    got = np.concatenate([s.forward([t])[1] for t in ids])
    rows_close(got, want, TOL[dtype], "token by token")
    s.reset()
    arg, lg = s.forward(ids, np.arange(24))
    rows_close(lg, want, TOL[dtype], "prompt")
    assert arg == int(np.argmax(lg[-1])) or dtype == "bfloat16"
    if dtype == "float32":
        s.reset()
        picks, _, _ = s.greedy(ids, 20)
        lg = follow(om, ids, picks)
        assert (lg.max(-1) - lg[np.arange(21), picks]).max() <= 1e-4 * lg.std()


def test_norm_and_head_alone(tg, folder):
    """Mixers that give nothing: the logits are the head on the normed embedding."""
    cfg = nm.config(50, 70, [nm.layer(nm.gla(1, 8, 8)), nm.layer(nm.latent(1, 8, 8, 8, 1.0))])
    path, om = folder("norm", cfg, seed=15, edit=zero_mixer)
    ids = np.arange(70, dtype=np.int32)
    want = om.norm("final.norm", om.t["embed"][ids]) @ om.t["head"].T
    model = tg.Transformer.from_dir(path, "float32")
    s = model.open_session(70)
    rows_close(s.forward(ids, ids)[1], want, F32_TOL, "head")
    assert s.position == 70
    s.reset()
    rows_close(np.concatenate([s.forward([t])[1] for t in ids]), want, F32_TOL, "head, token by token")


# ---- whole models ------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", nm.MODELS)
def test_prompts_and_decoding(tg, folder, name, dtype):
    """All logits of a prompt, the residual stream behind every block, and the same tokens one by one."""
    cfg = nm.MODELS[name]
    path, om = folder(name, cfg, seed=20)
    n = 140
    ids = ids_of(cfg, n, 5)
    taps = []
    want = om.step(om.state(), ids, taps)
    model = tg.Transformer.from_dir(path, dtype)
    assert model.architecture == "Madevik" and model.cfg.n_vocab == cfg["vocab"] and model.cfg.n_layers == len(cfg["layers"])
    s = model.open_session(n)
    loose = 0.0 if dtype == "float32" else 0.15
    arg, got = s.forward(ids, np.arange(n))
    rows_close(got, want, TOL[dtype], "prompt logits", loose)
    if dtype == "float32":
        assert arg == int(np.argmax(got[-1]))
        for l in range(len(cfg["layers"])):
            rows_close(s.tap(2 * l + 2, rows=n), taps[l], F32_TOL, f"layer {l}")
    s.reset()
    got = np.concatenate([s.forward([t])[1] for t in ids])
    rows_close(got, want, TOL[dtype], "token by token", loose)
    if dtype == "float32":
        for l in range(len(cfg["layers"])):
            rows_close(s.tap(2 * l + 2), taps[l][-1:], F32_TOL, f"layer {l}, last token")


PORTIONS = {"twos": [2] * 40, "ones_and_twos": [1, 2, 1, 1, 2, 3] * 8, "edges": [63, 1, 1, 63, 2, 64, 65], "growing": [2, 3, 5, 9, 17, 33, 65, 129],
            "then_single": [100] + [1] * 40, "around_64": [64, 2, 62, 66]}


@pytest.mark.parametrize("cut", PORTIONS)
@pytest.mark.parametrize("name", ["ragged", "flat"])
def test_portions(tg, folder, name, cut):
    cfg = nm.MODELS[name]
    path, om = folder(name, cfg, seed=20)
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


def test_wanted_places(tg, folder):
    cfg = nm.MODELS["ragged"]
    path, om = folder("ragged", cfg, seed=20)
    s = tg.Transformer.from_dir(path, "float32").open_session(300)
    ids = ids_of(cfg, 300, 7)
    _, all_ = s.forward(ids, np.arange(300))
    for want in ([0], [299], [0, 1, 64, 65, 298], []):
        s.reset()
        _, got = s.forward(ids, want)
        assert got.shape == (len(want), cfg["vocab"]) and np.array_equal(got, all_[want])


def test_sessions_used_again_and_side_by_side(tg, folder):
    """A reset session, a new session and sessions taken in turns give the same bits."""
    cfg = nm.MODELS["ragged"]
    path, _ = folder("ragged", cfg, seed=20)
    model = tg.Transformer.from_dir(path, "bfloat16")
    runs = [ids_of(cfg, n, 30 + n) for n in (90, 7, 131)]
    cuts = [[40, 1, 1, 48], [3, 1, 3], [2, 100, 1, 28]]

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
    got, at = [[] for _ in runs], [0] * 3
    for step in range(4):
        for i in range(3):
            if step < len(cuts[i]):
                k = cuts[i][step]
                got[i].append(sess[i].forward(runs[i][at[i]:at[i] + k], np.arange(k))[1])
                at[i] += k
    for g, w in zip(got, fresh):
        assert np.array_equal(np.concatenate(g), w)


# ---- keys far away ---------------------------------------------------------------------------------------------------------------
def standout_case(folder, kind):
    """A one-layer model and a prompt maker: the last token's query meets one stand-out key, everything else low ones."""
    if kind == "latent":
        cfg = nm.config(64, 211, [nm.layer(nm.latent(2, 32, 32, 48, 1.0))])
    else:
        cfg = nm.config(64, 211, [nm.layer(nm.gla(2, 32, 32, 16.0))])
    path, om = folder(("standout", kind), cfg, seed=41, gain=2.0, decay=(9.0, 0.3))
    h = om.norm("l0.norm1", om.t["embed"])
    t, q_tok = om.t, 17
    q = (t["l0.mix.q"] @ h[q_tok]).reshape(2, 32)
    if kind == "latent":
        c = layers.rms_norm(h @ t["l0.mix.dkv"].T, t["l0.mix.dkv.norm"], cfg["norm"]["eps"])
        k = (c @ t["l0.mix.uk"].T).reshape(-1, 2, 32)
        score = np.einsum("hd,vhd->v", q, k)
    else:
        k = (h @ t["l0.mix.k"].T).reshape(-1, 2, 32)
        score = np.abs(np.einsum("hd,vhd->vh", q, k)).sum(-1)
    order = np.argsort(score)
    low = order[:60]
    low = low[low != q_tok]

    def prompt(n, at, seed=0):
        ids = np.random.default_rng(seed).choice(low, n).astype(np.int32)
        ids[-1] = q_tok
        plain = ids.copy()
        ids[at] = order[-1]
        return ids, plain

    return cfg, path, om, prompt


@pytest.mark.parametrize("kind", ["latent", "gla"])
@pytest.mark.parametrize("at", [0, 1, 15, 16, 31, 63, 64, 65, 127, 128, 190, 191, 192, 254, 255])
def test_one_key_that_stands_out(tg, folder, kind, at):
    """A single key at the edges of tiles and chunks: seen from the last place of a prompt and from a decoded token."""
    cfg, path, om, prompt = standout_case(folder, kind)
    n = 257
    ids, plain = prompt(n, at)
    want, without = om.step(om.state(), ids)[-1], om.step(om.state(), plain)[-1]
    assert normrel(without, want) > 2e-2      # the key shows, 2000 times the bound
    model = tg.Transformer.from_dir(path, "float32")
    s = model.open_session(n)
    rows_close(s.forward(ids)[1], want[None], F32_TOL, f"prompt, key {at}")
    s.reset()
    s.forward(ids[:-1])
    rows_close(s.forward(ids[-1:])[1], want[None], F32_TOL, f"decoded, key {at}")
    s.reset()
    s.forward(ids[:at + 1])
    if at + 1 < n - 2:
        s.forward(ids[at + 1:-2])
    rows_close(s.forward(ids[max(at + 1, n - 2):])[1], want[None], F32_TOL, f"portions cut behind key {at}")


@pytest.mark.parametrize("n", [1023, 1024, 1025, 1100])
def test_decoding_where_the_partials_need_a_fold(tg, folder, n):
    """Around 1024 keys a decode step of the latent attention starts to fold its partials in a launch of its own."""
    cfg, path, om, prompt = standout_case(folder, "latent")
    ids, _ = prompt(n, 5)
    taps = []
    t = om.t
    h = om.norm("l0.norm1", t["embed"][ids])
    # the last query only (the oracle's full prompt is quadratic): fill the cache, then one step
    cache = list(layers.rms_norm(h[:-1] @ t["l0.mix.dkv"].T, t["l0.mix.dkv.norm"], cfg["norm"]["eps"]))
    want = om.step([cache], ids[-1:], taps)
    s = tg.Transformer.from_dir(path, "float32").open_session(n)
    s.forward(ids[:-1])
    rows_close(s.forward(ids[-1:])[1], want, F32_TOL, f"{n} keys")


def test_long_context_over_several_passes(tg, folder):
    """16,500 tokens: several passes of a prefill, more than 64 keys per workgroup in a decode step.  The last query against
    the oracle (latent attention) and decoding against a portion (both mixers)."""
    cfg, path, om, prompt = standout_case(folder, "latent")
    n = 16500
    ids, _ = prompt(n, 4095)
    t = om.t
    h = om.norm("l0.norm1", t["embed"][ids])
    cache = list(layers.rms_norm(h[:-1] @ t["l0.mix.dkv"].T, t["l0.mix.dkv.norm"], cfg["norm"]["eps"]))
    want = om.step([cache], ids[-1:])
    for dtype in ("float32", "bfloat16"):
        s = tg.Transformer.from_dir(path, dtype).open_session(n)
        whole = s.forward(ids)[1]
        rows_close(whole, want, TOL[dtype], "prompt")
        s.reset()
        s.forward(ids[:-1])
        rows_close(s.forward(ids[-1:])[1], want, TOL[dtype], "decoded")
    cfg, path, om, prompt = standout_case(folder, "gla")
    ids, _ = prompt(9000, 4096)
    s = tg.Transformer.from_dir(path, "float32").open_session(9000)
    whole = s.forward(ids)[1]
    s.reset()
    s.forward(ids[:5001])
    s.forward(ids[5001:-40])
    for tok in ids[-40:]:
        last = s.forward([tok])[1]
    rows_close(last, whole, 1e-4, "9000 tokens of recurrence")


# ---- generation -------------------------------------------------------------------------------------------------------------------
def follow(om, prompt, ids):
    """The oracle's logits at every place where `ids` were picked."""
    st = om.state()
    out = [om.step(st, prompt)[-1]]
    for t in ids[:-1]:
        out.append(om.step(st, [t])[-1])
    return np.array(out)


@pytest.mark.parametrize("name", ["ragged", "flat", "tiny"])
def test_greedy_generation(tg, folder, name):
    """tg_generate_greedy (prefill, picks and decode steps chained on the device): every pick is the oracle's, or one whose
    logit is within rounding of the oracle's best."""
    cfg = nm.MODELS[name]
    path, om = folder(name, cfg, seed=20)
    prompt = ids_of(cfg, 30, 8)
    model = tg.Transformer.from_dir(path, "float32")
    s = model.open_session(30 + 200)
    ids, _, _ = s.greedy(prompt, 199)
    assert s.position == 229 and ids.shape == (200,)
    lg = follow(om, prompt, ids)
    spread = lg.std()
    gap = lg.max(-1) - lg[np.arange(200), ids]
    assert gap.max() <= 1e-4 * max(spread, 1e-3), float(gap.max())
    # in two batches, and behind a prompt of one token, the same
    s.reset()
    tok, _ = s.prefill(prompt, want_logits=False)
    s.decode_enqueue(50)
    s.decode_enqueue(149)
    assert np.array_equal(s.read_ids(200), ids)
    with pytest.raises(tg.TgError):
        s.decode_enqueue(2)                 # one position is left
    s2 = model.open_session(8)
    one, _, _ = s2.greedy(prompt[:1], 6)
    lg = follow(om, prompt[:1], one)
    assert (lg.max(-1) - lg[np.arange(7), one]).max() <= 1e-4 * max(lg.std(), 1e-3)


def test_captured_steps_equal_stream_launches(tg, folder):
    """Decode steps replayed from captured graphs (position read on the device, launches sized for a bound of the context):
    the same picks, logits and residual stream as stream launches, over many replays, with prefills and other work between
    them and across a change of the bound."""
    cfg = nm.MODELS["flat"]
    path, om = folder("flat", cfg, seed=20)
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
            out.append(s.tap(2 * len(cfg["layers"]))[0].tolist())
            out.append(s.decode(5)[1].tolist())
        runs[mode] = out
    assert runs[0] == runs[1]
    tg.check(tg.lib().tg_set_graphs(-1))


def test_sampled_generation(tg, folder):
    """The min-p sampler on a vocabulary that is no multiple of its blocks: every draw lies where the cumulative
    distribution of the oracle's logits crosses the uniform number."""
    cfg = nm.MODELS["ragged"]
    path, om = folder("ragged", cfg, seed=20)
    prompt = ids_of(cfg, 20, 9)
    s = tg.Transformer.from_dir(path, "float32").open_session(80)
    randf = np.random.default_rng(1).random(41, dtype=np.float32)
    for minp, temp in ((0.0, 1.0), (0.0, 0.5)):
        s.reset()
        ids, _, _ = s.generate(prompt, 40, minp, temp, randf)
        lg = follow(om, prompt, ids) / temp
        p = np.exp(lg - lg.max(-1, keepdims=True))
        c = np.cumsum(p / p.sum(-1, keepdims=True), -1)
        for i, t in enumerate(ids):
            lo = c[i, t - 1] if t else 0.0
            assert lo - 1e-4 <= randf[i] <= c[i, t] + 1e-4, (i, int(t))
        assert np.unique(ids).size > 5
    s.reset()
    greedy, _, _ = s.generate(prompt, 40, 1.5, 1.0, randf)   # minp >= 1: argmax
    s.reset()
    assert np.array_equal(greedy, s.greedy(prompt, 40)[0])


def test_prefill_and_decode_entry_points(tg, folder):
    cfg = nm.MODELS["ragged"]
    path, om = folder("ragged", cfg, seed=20)
    ids = ids_of(cfg, 40, 10)
    want = om.step(om.state(), ids)
    s = tg.Transformer.from_dir(path, "float32").open_session(64)
    tok, lg = s.prefill(ids[:30])
    rows_close(lg[None], want[29:30], F32_TOL, "prefill")
    with pytest.raises(tg.TgError):
        s.prefill(ids[:2])                  # not empty
    for i in range(30, 40):
        tok, lg = s.decode(ids[i])
        rows_close(lg[None], want[i:i + 1], F32_TOL, f"decode {i}")
        assert tok == int(np.argmax(lg))
    s.release_workspace()
    s.reset()
    rows_close(s.forward(ids, [39])[1], want[39:], F32_TOL, "after release")


def test_gemma_sessions_take_portions(tg, weight_images, oracle):
    """The same entry points on a Gemma model: portions of a sequence against its whole-prompt prefill."""
    model = tg.Transformer(tg.named_config("270m", 2))
    model.read_weights_mem(weight_images("270m", 2, 21))
    ids = np.random.default_rng(0).integers(0, 262144, 24).astype(np.int32)
    s = model.open_session(100)
    tok, lg = s.forward(ids)
    s.reset()
    s.forward(ids[:20])
    tok2, lg2 = s.forward(ids[20:], [1, 3])
    assert model.architecture == "Gemma3" and s.position == 24
    assert normrel(lg2[1], lg[0]) < 8e-3 and lg2.shape == (2, 262144)


# ---- folders that are wrong ----------------------------------------------------------------------------------------------------
def test_folder_errors(tg, tmp_path):
    cfg = nm.config(16, 20, [nm.layer(nm.gla(1, 8, 8), nm.moe(2, 1, 8)), nm.layer(nm.latent(1, 8, 8, 8, 1.0))])
    t = nm.weights(cfg, 1)
    n = [0]

    def broken(edit_cfg=None, edit_t=None, raw=None):
        c, w = json.loads(json.dumps(cfg)), dict(t)
        if edit_cfg:
            edit_cfg(c)
        if edit_t:
            edit_t(w)
        n[0] += 1
        p = nm.write(tmp_path / str(n[0]), c, w)
        if raw:
            raw(p)
        with pytest.raises(tg.TgError) as e:
            tg.Transformer.from_dir(p)
        return str(e.value)

    assert "unknown architecture" in broken(lambda c: c.update(architecture="Nobody"))
    assert "'tau'" in broken(lambda c: c["layers"][0]["mixer"].pop("tau"))
    assert "unknown mixer" in broken(lambda c: c["layers"][0].update(type="other"))
    assert "unknown feed-forward" in broken(lambda c: c["layers"][0]["mlp"].update(kind="dense"))
    assert "l0.mix.q" in broken(edit_t=lambda w: w.pop("l0.mix.q"))
    assert "another shape" in broken(edit_t=lambda w: w.update({"l1.mix.uk": w["l1.mix.uk"][:, :-1]}))
    assert "another shape" in broken(lambda c: c.update(width=17))
    assert "more experts" in broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=3))
    assert "differs from the layer" in broken(lambda c: c["layers"][1].update(weights_of=0))
    assert "shares the weights" in broken(lambda c: c["layers"][1].update(weights_of=1))

    def cut(p):
        f = os.path.join(p, "model.safetensors")
        data = open(f, "rb").read()
        open(f, "wb").write(data[:-64])
    assert "outside the file" in broken(raw=cut)
    assert "JSON" in broken(raw=lambda p: open(os.path.join(p, "config.json"), "w").write("{\"architecture\": "))
    with pytest.raises(tg.TgError):
        tg.Transformer.from_dir(str(tmp_path / "nowhere"))
    p = nm.write(tmp_path / "good", cfg, t)
    model = tg.Transformer.from_dir(p)
    s = model.open_session(4)
    for bad in ([20], [-1], [1, 2, 3, 4, 5], []):
        with pytest.raises(tg.TgError):
            s.forward(np.array(bad, np.int32), [])
    with pytest.raises(tg.TgError):
        s.forward([1, 2], [1, 1])
    with pytest.raises(tg.TgError):
        s.kv(0)
    s.forward([1, 2, 3])
    model.free()
    with pytest.raises(tg.TgError):
        s.forward([1])
    with pytest.raises(tg.TgError):
        s.reset()


# ---- programs ---------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run(tg, folder, tmp_path, dtype):
    cfg = nm.MODELS["ragged"]
    path, om = folder("ragged", cfg, seed=20)
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
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(len(steps))]
    wa, wb = om.step(om.state(), a), om.step(om.state(), b)
    want = {0: wa[[0, 29]], 2: wa[[32]], 3: wa[[49]], 4: wb[[2, 8]], 5: wa[[4]]}
    assert sorted(os.listdir(out)) == sorted(f"{i}.f32" for i in want)
    for i, w in want.items():
        got = np.fromfile(out / f"{i}.f32", "<f4").reshape(-1, cfg["vocab"])
        rows_close(got, w, TOL[dtype], f"step {i}", 0.0 if dtype == "float32" else 0.5)


def test_command_line(tg, folder):
    """host/gemma on a model folder: the ids of Session.generate."""
    cfg = nm.MODELS["ragged"]
    path, om = folder("ragged", cfg, seed=20)
    exe = os.path.join(ROOT, "tiny-gemma_amd", "host", "gemma")
    assert os.path.exists(exe), "host/gemma is not built: run __graft_entry__.build()"
    prompt = ids_of(cfg, 12, 60)
    env = dict(os.environ, LD_LIBRARY_PATH=os.path.join(ROOT, "tiny-gemma_amd") + ":" + os.environ.get("LD_LIBRARY_PATH", ""))

    def run(*args):
        return subprocess.run([exe, "--model_dir", path, *args], capture_output=True, text=True, env=env, timeout=100)

    text = " ".join(str(t) for t in prompt)
    r = run("--dtype", "float32", "--prompt_ids", text, "--n_dec", "20")
    assert r.returncode == 0, r.stderr
    ids = [int(x) for x in r.stdout.split("Prompt length: 12\n")[1].split("\n")[0].split()]
    s = tg.Transformer.from_dir(path, "float32").open_session(40)
    assert ids == s.greedy(prompt, 20)[0].tolist()
    assert "Decode Tok/s" in r.stdout
    a = run("--prompt_ids", text, "--n_dec", "20", "--minp", "0.0", "--seed", "7")
    b = run("--prompt_ids", text, "--n_dec", "20", "--minp", "0.0", "--seed", "7")
    assert a.returncode == 0 and a.stdout.split("\n\n")[0] == b.stdout.split("\n\n")[0] and a.stdout.split("\n\n")[0] != r.stdout.split("\n\n")[0]
    assert run("--prompt_ids", "5 six").returncode == 1
    assert run("--prompt_ids", "5 101").returncode == 1
    assert run("--dtype", "float16", "--prompt_ids", "5").returncode == 1
