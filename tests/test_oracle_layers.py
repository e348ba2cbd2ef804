"""CPU: the plain statements of the layer-list mechanisms (oracle/layers.py) against other forms of the same equations."""
import numpy as np
import pytest

import net_models as nm
from oracle import layers


def test_bf16_round_trip_and_safetensors(tmp_path):
    a = layers.round_bf16(np.array([0.0, 1.0, -2.5, 1.00390625, 3e38, 1e-30], np.float32))
    assert np.array_equal(layers.round_bf16(a), a)
    assert layers.round_bf16(np.float32(1.0 + 2 ** -8)) == 1.0          # half way: to even
    assert layers.round_bf16(np.float32(1.0 + 3 * 2 ** -8)) == np.float32(1.0 + 2 ** -6)
    t = {"m": a[:6].reshape(2, 3), "s": a[2].reshape(())}
    layers.write_safetensors(tmp_path / "x.safetensors", t)
    back = layers.read_safetensors(tmp_path / "x.safetensors")
    assert set(back) == set(t) and all(np.array_equal(back[k], t[k]) and back[k].shape == t[k].shape for k in t)


def test_dynamic_tanh_and_rms():
    x = np.array([0.0, 1.0, -30.0, 0.25])
    assert np.allclose(layers.dynamic_tanh(x, 2.0, np.array([1.0, 2.0, 3.0, 1.0]), np.array([0.5, 0.0, 1.0, 0.0])),
                       [0.5, 2 * np.tanh(2.0), 1.0 - 3.0, np.tanh(0.5)])
    y = layers.rms_norm(np.array([3.0, 4.0]), np.ones(2), 0.0)
    assert np.allclose(y, np.array([3.0, 4.0]) / np.sqrt(12.5))
    assert np.allclose(layers.rms_norm(np.zeros(4), np.ones(4), 1e-5), 0.0)


def test_sigmoids_far_out():
    z = np.array([-800.0, -1.0, 0.0, 1.0, 800.0])
    assert np.allclose(layers.sigmoid(z), [0.0, 1 / (1 + np.e), 0.5, np.e / (1 + np.e), 1.0])
    assert np.allclose(layers.log_sigmoid(z), [-800.0, -np.log1p(np.e), -np.log(2.0), -np.log1p(np.exp(-1.0)), 0.0])


def test_gla_recurrence_equals_the_sum_over_pairs():
    """o_i = sum_{j <= i} (sum_d q_id k_jd prod_{j < s <= i} alpha_sd) v_j, from the projections directly."""
    cfg = nm.config(24, 11, [nm.layer(nm.gla(2, 5, 3, 2.0))])
    m = layers.LayerModel(cfg, nm.weights(cfg, 1, rank=4))
    rng = np.random.default_rng(0)
    h = rng.standard_normal((13, 24))
    got = m.mixer(0, h, m.state()[0])
    t = m.t
    q = (h @ t["l0.mix.q"].T).reshape(13, 2, 5) / np.sqrt(5)
    k = (h @ t["l0.mix.k"].T).reshape(13, 2, 5)
    v = (h @ t["l0.mix.v"].T).reshape(13, 2, 3)
    z = h @ t["l0.mix.a1"].T @ t["l0.mix.a2"].T + t["l0.mix.a2.b"]
    la = np.log(1 / (1 + np.exp(-z))).reshape(13, 2, 5) / 2.0
    want = np.zeros((13, 2, 3))
    for i in range(13):
        for j in range(i + 1):
            w = np.exp(la[j + 1:i + 1].sum(0))
            want[i] += (q[i] * k[j] * w).sum(-1, keepdims=True) * v[j]
    want = want / np.sqrt((want ** 2).mean(-1, keepdims=True) + 1e-5) * t["l0.mix.norm"]
    g = h @ t["l0.mix.g"].T
    want = (want.reshape(13, 6) * g / (1 + np.exp(-g))) @ t["l0.mix.o"].T
    assert np.allclose(got, want, atol=1e-10)


def test_latent_attention_equals_full_matrices():
    cfg = nm.config(24, 11, [nm.layer(nm.latent(3, 5, 4, 6, 0.7))])
    m = layers.LayerModel(cfg, nm.weights(cfg, 2))
    h = np.random.default_rng(0).standard_normal((9, 24))
    got = m.mixer(0, h, [])
    t = m.t
    c = h @ t["l0.mix.dkv"].T
    c = c / np.sqrt((c ** 2).mean(-1, keepdims=True) + 1e-5) * t["l0.mix.dkv.norm"]
    q = (h @ t["l0.mix.q"].T).reshape(9, 3, 5)
    k = (c @ t["l0.mix.uk"].T).reshape(9, 3, 5)
    v = (c @ t["l0.mix.uv"].T).reshape(9, 3, 4)
    s = np.einsum("ihd,jhd->hij", q, k) * 0.7
    s = np.where(np.tril(np.ones((9, 9), bool)), s, -np.inf)
    p = np.exp(s - s.max(-1, keepdims=True))
    p /= p.sum(-1, keepdims=True)
    o = np.einsum("hij,jhv->ihv", p, v) / (1 + np.exp(-(h @ t["l0.mix.g"].T)))[:, :, None]
    assert np.allclose(got, o.reshape(9, 12) @ t["l0.mix.o"].T, atol=1e-12)


def test_routing_uses_the_correction_for_the_choice_only():
    chosen, w = layers.route(np.array([0.9, 0.5, 0.4, 0.1]), np.array([-1.0, 0.0, 0.2, 0.0]), 2, 3.0)
    assert chosen == [2, 1] and np.allclose(w, np.array([0.4, 0.5]) / 0.9 * 3.0)
    chosen, _ = layers.route(np.array([0.5, 0.5, 0.5]), np.zeros(3), 2, 1.0)
    assert chosen == [0, 1]                                             # ties: the lower index
    _, w = layers.route(np.zeros(3), np.zeros(3), 3, 1.0)
    assert np.allclose(w, 0.0)


def test_rotation_depends_on_the_distance_only():
    rng = np.random.default_rng(0)
    for interleaved in (True, False):
        q, k = rng.standard_normal((2, 12))
        s = [layers.rotate(q, p + 7, 8, 50.0, interleaved) @ layers.rotate(k, p, 8, 50.0, interleaved) for p in (0, 3, 40)]
        assert np.allclose(s, s[0])
        r = layers.rotate(q, 5, 8, 50.0, interleaved)
        assert np.array_equal(r[8:], q[8:]) and np.isclose(np.linalg.norm(r), np.linalg.norm(q)) and not np.allclose(r[:8], q[:8])
    x = rng.standard_normal(8)
    pairs = np.arange(8).reshape(4, 2).T.reshape(-1)          # interleaved pairs brought side by side in halves
    assert np.allclose(layers.rotate(x, 9, 8, 50.0, True)[pairs], layers.rotate(x[pairs], 9, 8, 50.0, False))
    z = x[0] + 1j * x[1]                                      # the first pair turns by the position itself
    assert np.allclose(layers.rotate(x, 2, 8, 50.0, True)[:2], [(z * np.exp(2j)).real, (z * np.exp(2j)).imag])


def banded_softmax(s, window):
    n = s.shape[-1]
    i, j = np.mgrid[:n, :n]
    s = np.where((i - j >= 0) & (i - j < window), s, -np.inf)
    p = np.exp(s - s.max(-1, keepdims=True))
    return p / p.sum(-1, keepdims=True)


def test_rotated_latent_attention_equals_full_matrices():
    cfg = nm.tutelix(24, 11, [nm.layer(nm.rot_latent(3, 5, 4, 7, 9, 6, 4, 0.7, 30.0))])
    m = layers.model_of(cfg, nm.weights(cfg, 2))
    h = np.random.default_rng(0).standard_normal((9, 24))
    got = m.mixer(0, h, [])
    t = {k.split("mix.")[-1]: v for k, v in m.t.items()}
    cq = h @ t["dq"].T
    q = (cq / np.sqrt((cq ** 2).mean(-1, keepdims=True) + 1e-5) * t["dq.norm"] @ t["uq"].T).reshape(9, 3, 9)
    kv = h @ t["dkv"].T
    c = kv[:, :6] / np.sqrt((kv[:, :6] ** 2).mean(-1, keepdims=True) + 1e-5) * t["dkv.norm"]
    k = np.concatenate([(c @ t["uk"].T).reshape(9, 3, 5), np.repeat(kv[:, None, 6:], 3, 1)], -1)
    turn = np.exp(1j * np.arange(9)[:, None] * 30.0 ** (-np.arange(0, 4, 2) / 4))
    for x in (q, k):
        z = (x[..., 5::2] + 1j * x[..., 6::2]) * turn[:, None]
        x[..., 5::2], x[..., 6::2] = z.real, z.imag
    p = banded_softmax(np.einsum("ihd,jhd->hij", q, k) * 0.7, 4)
    o = np.einsum("hij,jhv->ihv", p, (c @ t["uv"].T).reshape(9, 3, 7))
    assert np.allclose(got, o.reshape(9, 21) @ t["o"].T, atol=1e-12)


def test_attention_on_its_keys_equals_full_matrices():
    cfg = nm.tutelix(24, 11, [nm.layer(nm.key_values(6, 2, 7, 4, 3, 0.7, 30.0))])
    m = layers.model_of(cfg, nm.weights(cfg, 2))
    h = np.random.default_rng(0).standard_normal((9, 24))
    got = m.mixer(0, h, [])
    t = {k.split("mix.")[-1]: v for k, v in m.t.items()}
    q, v = (h @ t["q"].T + t["q.b"]).reshape(9, 6, 7), (h @ t["k"].T + t["k.b"]).reshape(9, 2, 7)
    k = v.copy()
    turn = np.exp(1j * np.arange(9)[:, None] * 30.0 ** (-np.arange(0, 4, 2) / 4))[:, None]
    for x in (q, k):
        z = (x[..., :2] + 1j * x[..., 2:4]) * turn
        x[..., :2], x[..., 2:4] = z.real, z.imag
    own = np.array([0, 0, 0, 1, 1, 1])
    p = banded_softmax(np.einsum("ihd,jhd->hij", q, k[:, own]) * 0.7, 3)
    assert np.allclose(got, np.einsum("hij,jhv->ihv", p, v[:, own]).reshape(9, 42) @ t["o"].T, atol=1e-12)


def test_short_convolution_is_causal():
    rng = np.random.default_rng(0)
    x, w, past = rng.standard_normal((10, 3)), rng.standard_normal((3, 4)), []
    got = np.array([layers.short_conv(v, past, w) for v in x])
    want = np.stack([np.convolve(x[:, c], w[c, ::-1])[:10] for c in range(3)], -1)
    assert np.allclose(got, want)
    assert np.allclose(layers.short_conv(x[0], [], w), x[0] * w[:, -1])


def test_gated_delta_rule_equals_its_transition_matrices():
    """S_t = (1 - beta k k^T) diag(g) S_(t-1) + beta k v^T, and the state of a portion is carried to the next."""
    cfg = nm.tutelix(24, 11, [nm.layer(nm.delta(4, 2, 5, 3, 1))])
    m = layers.model_of(cfg, nm.weights(cfg, 1, rank=4, gate_rank=3))
    h = np.random.default_rng(0).standard_normal((12, 24))
    st = m.state()[0]
    got = np.concatenate([m.mixer(0, h[:5], st), m.mixer(0, h[5:], st)])
    t = {k.split("mix.")[-1]: v for k, v in m.t.items()}

    def silu(z):
        return z / (1 + np.exp(-z))
    q, k, v = (silu(h @ t[n].T * t[n + ".conv"][:, 0]) for n in "qkv")
    q, k, v = q.reshape(12, 2, 5), k.reshape(12, 2, 5), v.reshape(12, 4, 3)
    q, k = (x / np.sqrt((x ** 2).sum(-1, keepdims=True) + 1e-6) for x in (q, k))
    beta = 1 / (1 + np.exp(-h @ t["b"].T))
    z = (h @ t["a1"].T @ t["a2"].T + t["dt_bias"]).reshape(12, 4, 5)
    g = np.exp(-np.exp(t["A_log"])[:, None] * np.log1p(np.exp(z)))
    S, want = np.zeros((4, 5, 3)), np.zeros((12, 4, 3))
    for i in range(12):
        for a in range(4):
            kk = k[i, a // 2]
            S[a] = (np.eye(5) - beta[i, a] * np.outer(kk, kk)) @ np.diag(g[i, a]) @ S[a] + beta[i, a] * np.outer(kk, v[i, a])
            o = q[i, a // 2] / np.sqrt(5) @ S[a]
            want[i, a] = o / np.sqrt((o ** 2).mean() + 1e-5) * t["norm"]
    want = want.reshape(12, 12) / (1 + np.exp(-(h @ t["g1"].T @ t["g2"].T)))
    assert np.allclose(got, want @ t["o"].T, atol=1e-10)


def test_gelu_is_the_exact_one():
    z = np.array([-30.0, -1.0, 0.0, 0.5, 30.0])
    assert np.allclose(layers.gelu(z), [0.0, -0.15865525393145707, 0.0, 0.34573123063700656, 30.0], atol=1e-15)


def test_looped_layers_equal_layers_written_out():
    """A run of layers passed three times has the weights once and a state for each pass."""
    ls = [nm.layer(nm.delta(2, 1, 5, 3, 2), nm.dense(8)), nm.layer(nm.key_values(2, 1, 6, 4, 3, 0.7)), nm.layer(nm.rot_latent(2, 5, 4, 3, 6, 7, 4, 0.5), nm.dense(5))]
    cfg = nm.tutelix(16, 11, ls, loop=(1, 3, 3))
    t = nm.weights(cfg, 5)
    flat = nm.tutelix(16, 11, [ls[0]] + ls[1:] * 3, loop=(0, 1, 1))
    t2 = {k: v for k, v in t.items() if not k.startswith(("l1.", "l2."))}
    for k, v in t.items():
        if k.startswith(("l1.", "l2.")):
            t2.update({f"l{int(k[1]) + 2 * i}{k[2:]}": v for i in range(3)})
    a, b = layers.model_of(cfg, t), layers.model_of(flat, t2)
    assert a.runs() == [0, 1, 2, 1, 2, 1, 2] and len(a.state()) == 7
    ids = np.random.default_rng(4).integers(0, 11, 12)
    assert np.allclose(a.step(a.state(), ids), b.step(b.state(), ids), atol=1e-12)


@pytest.mark.parametrize("name", ["ragged", "tiny", "mixed", "ones"])
def test_portions_of_the_oracle_agree(name):
    cfg = nm.MODELS.get(name) or nm.TUTELIX[name]
    m = layers.model_of(cfg, nm.weights(cfg, 3))
    ids = np.random.default_rng(4).integers(0, cfg["vocab"], 12)
    whole = m.step(m.state(), ids)
    st = m.state()
    cut = np.concatenate([m.step(st, ids[a:b]) for a, b in ((0, 5), (5, 6), (6, 12))])
    assert np.allclose(whole, cut, atol=1e-12)


def test_random_model_dir_is_readable(tmp_path):
    import __graft_entry__ as ge
    import importlib
    ge.load_package()
    w = importlib.import_module("tiny_gemma_amd.weights")
    cfg = nm.MODELS["ragged"]
    w.random_model_dir(str(tmp_path / "m"), cfg, 5, decay_rank=3, block=1 << 12)
    m = layers.LayerModel.from_dir(str(tmp_path / "m"))
    assert np.isfinite(m.step(m.state(), [1, 2, 3])).all()
    assert sum(k.startswith("l3.") or k.startswith("l4.") for k in m.t) == 0   # shared layers have no tensors
    w.random_model_dir(str(tmp_path / "t"), nm.TUTELIX["mixed"], 5, decay_rank=3, block=1 << 12, gate_rank=4)
    m = layers.LayerModel.from_dir(str(tmp_path / "t"))
    assert isinstance(m, layers.TutelixModel) and np.isfinite(m.step(m.state(), [1, 2, 3])).all()
