"""The float64 restatement of Netinex's mechanisms against closed forms and independent formulations, and what
of the model class can be checked without a GPU."""
import ctypes as C
import json
import math
import os

import numpy as np
import pytest

from conftest import load_pkg
import netinex_models as xm
import nezavik_models as nm
from oracle import netinex_oracle as nx


def test_tanh_norm_and_softcap():
    x = np.array([[-50.0, -0.1, 0.0, 0.3, 50.0]])
    y = nx.tanh_norm(x, np.array([1, 2, 3, 4, 5.0]), np.array([0, 0, 7, 0, 1.0]), np.array(0.5))
    assert np.allclose(y, [[-1, 2 * math.tanh(-0.05), 7, 4 * math.tanh(0.15), 6]])
    assert np.allclose(nx.softcap(np.array([0.001, 1e9, -1e9]), 20.0), [0.001, 20, -20])


def test_rotation_keeps_lengths_and_depends_on_distance_only():
    rng = np.random.default_rng(0)
    rot = {"dims": 6, "base": 50.0}
    q, k = rng.standard_normal((1, 1, 9)), rng.standard_normal((1, 1, 9))
    for inter in (False, True):
        at = lambda x, p: nx.rotate(x, [p], rot, inter)[0, 0]
        assert np.allclose(at(q, 17)[6:], q[0, 0, 6:]) and np.allclose(at(q, 0), q[0, 0])
        assert np.isclose(np.linalg.norm(at(q, 17)), np.linalg.norm(q))
        assert np.isclose(at(q, 30) @ at(k, 21), at(q, 9) @ at(k, 0))
    # the two layouts are one rotation under a permutation of the dimensions
    perm = [0, 2, 4, 1, 3, 5, 6, 7, 8]
    assert np.allclose(nx.rotate(q, [5], rot, True)[..., perm], nx.rotate(q[..., perm], [5], rot, False))
    # one pair by hand: complex multiplication
    z = (q[0, 0, 1] + 1j * q[0, 0, 4]) * np.exp(1j * 5 * 50.0 ** (-2 / 6))
    assert np.allclose(nx.rotate(q, [5], rot, False)[0, 0, [1, 4]], [z.real, z.imag])


def test_yarn_frequencies():
    rot = {"dims": 64, "base": 10000.0, "scaling": {"factor": 16.0, "original": 4096, "fast": 32.0, "slow": 1.0}}
    f, gain = nx.frequencies(rot)
    plain, one = nx.frequencies({"dims": 64, "base": 10000.0})
    assert one == 1.0 and np.isclose(gain, 0.1 * math.log(16) + 1)
    ratio = f / plain
    turns = 4096 * plain / (2 * math.pi)
    assert np.allclose(ratio[turns > 45], 1) and np.allclose(ratio[turns < 0.7], 1 / 16)
    assert (np.diff(ratio) <= 1e-12).all() and ((ratio > 1 / 16 + 1e-6) & (ratio < 1 - 1e-6)).sum() > 5
    # both ends of the ramp at one place
    f, _ = nx.frequencies({"dims": 8, "base": 10.0, "scaling": {"factor": 2.0, "original": 1, "fast": 9.0, "slow": 8.0}})
    assert np.allclose(f[1:] * 2, 10.0 ** (-np.arange(1, 4) / 4)) and np.isclose(f[0], 1.0)


def test_retention_equals_its_sum_over_the_past_and_continues_from_its_state():
    rng = np.random.default_rng(1)
    T, H, K, V = 9, 2, 3, 4
    q, k, v = rng.standard_normal((T, H, K)), rng.standard_normal((T, H, K)), rng.standard_normal((T, H, V))
    decay = [0.5, 0.97]
    o, S = nx.retention(q, k, v, decay)
    for h in range(H):
        for t in range(T):
            want = sum(decay[h] ** (t - s) * (q[t, h] @ k[s, h]) * v[s, h] for s in range(t + 1))
            assert np.allclose(o[t, h], want)
    oa, Sa = nx.retention(q[:4], k[:4], v[:4], decay)
    ob, Sb = nx.retention(q[4:], k[4:], v[4:], decay, Sa)
    assert np.allclose(np.concatenate([oa, ob]), o) and np.allclose(S, Sb)


def test_chunk_attention_restarts_at_every_chunk():
    rng = np.random.default_rng(2)
    T, H, G, size = 13, 4, 2, 5
    q, k, v = rng.standard_normal((T, H, 3)), rng.standard_normal((T, G, 3)), rng.standard_normal((T, G, 6))
    got = nx.chunk_attention(q, k, v, 0.7, size)
    for i in range(T):
        lo = i - i % size
        for h in range(H):
            s = 0.7 * k[lo:i + 1, h // 2] @ q[i, h]
            p = np.exp(s)
            assert np.allclose(got[i, h], p / p.sum() @ v[lo:i + 1, h // 2])
    assert np.allclose(nx.chunk_attention(q, k, v, 0.7, 1)[:, 3], v[:, 1])


def test_router_weighs_the_chosen_only():
    z = np.array([[0.0, 3.0, 1.0, 2.0], [1.0, 1.0, 1.0, -5.0]])
    ids, share = nx.route(z, 2)
    assert ids.tolist() == [[1, 3], [0, 1]]
    assert np.allclose(share, [[1 / (1 + math.exp(-1)), 1 / (1 + math.e)], [0.5, 0.5]])
    assert np.allclose(nx.margin(z, 2), [1.0, 0.0]) and nx.margin(z, 4)[0] == np.inf


def test_feed_forward_with_every_expert_is_a_weighted_sum():
    cfg = xm.config([xm.retention(mlp=xm.moe(experts=3, top=3))])
    w, p = xm.weights(cfg, 3), "l0.mlp"
    h = np.random.default_rng(4).standard_normal((5, cfg["width"]))
    z = np.exp(h @ nx.f64(w[p + ".router"]).T + w[p + ".router.b"])
    want = 0
    for e in range(3):
        g, u = (h @ nx.f64(w[f"{p}.e{e}.{n}"]).T for n in ("gate", "up"))
        want = want + (z / z.sum(1, keepdims=True))[:, e:e + 1] * ((g / (1 + np.exp(-g)) * u) @ nx.f64(w[f"{p}.e{e}.down"]).T)
    assert np.allclose(nx.feed_forward(h, w, p, cfg["layers"][0]["mlp"]), want)


def test_values_are_the_keys_as_projected():
    """A single position attends to itself: the mixer's output is W_o of its own keys, untouched by norm and
    rotation."""
    cfg = xm.config([xm.attention()])
    w, h = xm.weights(cfg, 5), np.random.default_rng(6).standard_normal((1, 72))
    k = (h @ nx.f64(w["l0.mix.k"]).T).reshape(2, 32)
    want = np.repeat(k, 2, axis=0).reshape(1, -1) @ nx.f64(w["l0.mix.o"]).T
    assert np.allclose(nx.mixer_attention(h, w, "l0.mix", cfg["layers"][0]["mixer"], 1e-5), want)


def test_test_models_route_by_wide_margins():
    """What lets the GPU tests compare 16-bit runs: no token of the models is near a tie."""
    cfg = xm.config([xm.retention(mlp=xm.moe()), xm.attention(mlp=xm.moe(experts=9, top=3))])
    w, margins = xm.weights(cfg, 21), []
    nx.forward(cfg, w, nm.tokens(cfg, 120, 2), margins=margins)
    assert len(margins) == 2 and min(m.min() for m in margins) > 0.05


# ---- product, no GPU needed ----------------------------------------------------------------------
@pytest.fixture(scope="module")
def lib():
    L = load_pkg("lib")
    L.load()
    return L


def _open(lib, path, flags=0):
    h = C.c_void_p()
    rc = lib.load().gptoss_engine_open(str(path).encode(), 2, 16, flags, 0, C.byref(h))
    assert rc != 0 or h.value
    return rc, lib.last_error()


def test_open_reports_what_is_wrong(lib, tmp_path):
    cfg = xm.config([xm.retention(), xm.attention(mlp=xm.moe())])
    d = tmp_path / "m"
    nm.save(d, cfg, xm.weights(cfg))
    for key in ("vocab", "width", "norm", "layers"):
        (d / "config.json").write_text(json.dumps({k: v for k, v in cfg.items() if k != key}))
        rc, msg = _open(lib, d)
        assert rc == 7 and f'"{key}"' in msg, msg
    (d / "config.json").write_text(json.dumps(cfg))
    for flag in (lib.ENGINE_MXFP4_EXPERTS, lib.ENGINE_NO_PREFILL, lib.ENGINE_SYNTHETIC | lib.ENGINE_PRECISE):
        assert _open(lib, d, flag)[0] == 6


def test_the_sources_of_the_class_leave_other_classes_out():
    b = load_pkg("build")
    names = {os.path.basename(s) for s in b.sources()}
    own = set(b.CORE) | set(b.MODELS["Netinex"])
    assert own <= names and not set(b.CORE) & set(b.MODELS["Netinex"])
    assert not own & {"gemm_mxfp4.hip", "model_gptoss.cpp", "model_nezavik.cpp", "attn_decode.hip"}
