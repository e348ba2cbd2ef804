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


@pytest.mark.parametrize("name", ["ragged", "tiny"])
def test_portions_of_the_oracle_agree(name):
    cfg = nm.MODELS[name]
    m = layers.LayerModel(cfg, nm.weights(cfg, 3))
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
