"""The float64 restatement of Nezavik's mechanisms against closed forms and independent formulations,
and what of the model class can be checked without a GPU."""
import ctypes as C
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from conftest import ROOT, load_pkg
import nezavik_models as nm
from oracle import nezavik_oracle as nz


def test_short_conv_is_a_causal_convolution():
    rng = np.random.default_rng(0)
    x, taps, bias = rng.standard_normal((9, 3)), rng.standard_normal((3, 4)), rng.standard_normal(3)
    y = nz.short_conv(x, taps, bias)
    for c in range(3):
        assert np.allclose(y[:, c], np.convolve(x[:, c], taps[c, ::-1])[:9] + bias[c])
    assert np.allclose(nz.short_conv(x, taps[:, -1:]), x * taps[:, -1])     # one tap: no memory


def test_delta_rule_stores_and_overwrites():
    """Orthonormal keys, full write strength, no decay: reading a key returns the last value written to it."""
    keys, vals = np.eye(4), np.random.default_rng(1).standard_normal((6, 1, 5))
    order = [0, 1, 2, 1, 3, 0]
    k = keys[order][:, None, :]
    q = keys[[0, 0, 1, 2, 1, 0]][:, None, :]
    one = np.ones((6, 1))
    o, S = nz.delta_rule(q, k, vals, one, np.ones((6, 1, 4)))
    for t, src in enumerate([0, 0, 1, 2, 3, 5]):                          # a read includes what its own token wrote
        assert np.allclose(o[t, 0], vals[src, 0])
    # beta = 0 writes nothing; a decay of 0 forgets before it reads
    o2, S2 = nz.delta_rule(q, k, vals, 0 * one, np.ones((6, 1, 4)), S)
    assert np.allclose(S2, S)
    g = np.ones((6, 1, 4))
    g[0, 0, 2] = 0.0                                                      # one channel forgets
    _, S3 = nz.delta_rule(q, k, vals, 0 * one, g, S)
    assert np.allclose(S3[0, 2], 0) and np.allclose(S3[0, 1], S[0, 1])


def test_recurrences_continue_from_their_state():
    rng = np.random.default_rng(2)
    q, k, v = (rng.standard_normal((10, 2, n)) for n in (3, 3, 4))
    beta, g = rng.uniform(size=(10, 2)), rng.uniform(size=(10, 2, 3))
    o, S = nz.delta_rule(q, k, v, beta, g)
    oa, Sa = nz.delta_rule(q[:4], k[:4], v[:4], beta[:4], g[:4])
    ob, Sb = nz.delta_rule(q[4:], k[4:], v[4:], beta[4:], g[4:], Sa)
    assert np.allclose(np.concatenate([oa, ob]), o) and np.allclose(S, Sb)


def test_state_space_equals_its_sum_over_the_past():
    rng = np.random.default_rng(3)
    T, H, P, N = 7, 2, 3, 4
    x, B, Cm = rng.standard_normal((T, H, P)), rng.standard_normal((T, H, N)), rng.standard_normal((T, H, N))
    dt, a_log, d = rng.uniform(0.1, 1, (T, H)), rng.standard_normal(H), rng.standard_normal(H)
    y, _ = nz.state_space(x, B, Cm, dt, a_log, d)
    for h in range(H):
        for t in range(T):
            want = d[h] * x[t, h]
            for s in range(t + 1):
                decay = np.exp(-np.exp(a_log[h]) * dt[s + 1:t + 1, h].sum())
                want = want + decay * dt[s, h] * (B[s, h] @ Cm[t, h]) * x[s, h]
            assert np.allclose(y[t, h], want)


def test_window_attention_equals_a_masked_softmax():
    rng = np.random.default_rng(4)
    T, H, G, W = 11, 4, 2, 5
    q, k, v = rng.standard_normal((T, H, 3)), rng.standard_normal((T, G, 3)), rng.standard_normal((T, G, 6))
    got = nz.window_attention(q, k, v, 0.7, W)
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    for h in range(H):
        s = np.where((i >= j) & (i - j < W), 0.7 * q[:, h] @ k[:, h // 2].T, -np.inf)
        p = np.exp(s - s.max(axis=1, keepdims=True))
        assert np.allclose(got[:, h], p / p.sum(axis=1, keepdims=True) @ v[:, h // 2])
    assert np.allclose(nz.window_attention(q, k, v, 0.7, 1)[:, 0], v[:, 0])    # only itself


def test_pointwise_functions():
    z = np.linspace(-40, 40, 801)
    assert np.allclose(nz.sigmoid(z) + nz.sigmoid(-z), 1)
    assert np.allclose(nz.softplus(z) - nz.softplus(-z), z)
    assert np.allclose(nz.silu(z), z * nz.sigmoid(z))
    assert np.array_equal(nz.relu_squared(np.array([-2.0, 0.0, 3.0])), [0, 0, 9])
    x = np.random.default_rng(5).standard_normal((3, 8))
    assert np.allclose(np.square(nz.over_rms(x, 0.0)).mean(axis=1), 1)
    assert np.allclose(np.linalg.norm(nz.unit_vectors(x), axis=1), 1, atol=1e-6)


def test_depth_average_weighs_layer_results_and_embedding():
    cfg = nm.config([nm.delta(ff=None), nm.delta(ff=None)])
    w = nm.weights(cfg, 6)
    for i in range(2):
        w[f"l{i}.mix.o"] = np.zeros_like(w[f"l{i}.mix.o"])      # every layer's result is its input
    w["l0.dwa"], w["l1.dwa"] = np.array([0.5, 2.0]), np.array([1.0, -3.0, 0.25])
    tok = nm.tokens(cfg, 4, 0)
    _, after = nz.forward(cfg, w, tok, want_layers=True)
    x0 = nz.f64(w["embed"])[tok] + nz.f64(w["pos"])[:4]
    assert np.allclose(after[0], 2.5 * x0)                      # X_1 = x0
    assert np.allclose(after[1], x0 - 3 * x0 + 0.25 * 2.5 * x0)  # X_1 is the result before the averaging


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


def test_registry_lists_the_model_classes(lib):
    names, i = [], 0
    while (n := lib.load().gptoss_model_name(i)) is not None:
        names.append(n.decode())
        i += 1
    assert sorted(names) == ["Netinex", "Nezavik", "gpt-oss"]


def test_open_reports_what_is_wrong(lib, tmp_path):
    assert _open(lib, tmp_path / "nowhere") == (7, f"engine_open: {tmp_path / 'nowhere'} does not exist")
    d = tmp_path / "m"
    d.mkdir()
    assert _open(lib, d)[0] == 7                                   # no config.json
    (d / "config.json").write_text("{ not json")
    assert "not a JSON object" in _open(lib, d)[1]
    (d / "config.json").write_text('{"architecture": "Unknown"}')
    assert 'no model class for architecture "Unknown"' in _open(lib, d)[1]
    cfg = nm.config([nm.delta()])
    (d / "config.json").write_text(json.dumps(cfg))
    assert "model.safetensors" in _open(lib, d)[1]
    (d / "model.safetensors").write_bytes(b"\x05\x00\x00\x00\x00\x00\x00\x00hello")
    assert "not a safetensors file" in _open(lib, d)[1]
    nm.save(d, cfg, nm.weights(cfg))
    for key in ("vocab", "width", "max_positions", "norm", "layers"):
        broken = {k: v for k, v in cfg.items() if k != key}
        (d / "config.json").write_text(json.dumps(broken))
        rc, msg = _open(lib, d)
        assert rc == 7 and f'"{key}"' in msg, msg
    (d / "config.json").write_text(json.dumps(cfg))
    assert _open(lib, d, lib.ENGINE_MXFP4_EXPERTS)[0] == 6          # flags of the other model class
    assert _open(lib, d, lib.ENGINE_SYNTHETIC | lib.ENGINE_PRECISE)[0] == 6
    (tmp_path / "x.bin").write_bytes(b"\x00" * 100)
    assert _open(lib, tmp_path / "x.bin")[0] == 7


def test_engine_entry_points_validate_arguments(lib):
    L = lib.load()
    p = C.cast((C.c_char * 64)(), C.c_void_p)
    assert L.gptoss_engine_step_logits(None, 1, p, p, p, 0, None, None) == 1
    assert L.gptoss_engine_slot_acquire(None, C.byref(C.c_int())) == 1
    assert L.gptoss_engine_slot_release(None, 0) == 1
    assert L.gptoss_engine_info(None, None) == 1
    assert L.gptoss_engine_open(None, 1, 1, 0, 0, C.byref(C.c_void_p())) == 1


def test_the_sources_of_one_model_class_link_without_the_others():
    """Core and class sources are disjoint, exist, and leave the other class's files out."""
    b = load_pkg("build")
    names = {os.path.basename(s) for s in b.sources()}
    own = set(b.CORE) | set(b.MODELS["Nezavik"])
    assert own <= names and not set(b.CORE) & set(b.MODELS["Nezavik"])
    assert not own & {"moe_layer.cpp", "moe_gemm.hip", "moe_route.hip", "gemm_mxfp4.hip", "model_gptoss.cpp", "attn_decode.hip"}


def test_command_line_help_needs_no_gpu():
    for cmd in (["--help"], ["generate", "--help"], ["trace", "--help"]):
        r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "gptoss")] + cmd, capture_output=True, text=True,
                           timeout=60)
        assert r.returncode == 0 and "usage" in r.stdout
