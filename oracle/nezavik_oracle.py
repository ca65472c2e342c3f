"""Plain float64 numpy restatement of the Nezavik decoder: one function per mechanism, a token loop
wherever the design has a recurrence, no caches and no batching.  Shares no code with the product.

TEST INFRASTRUCTURE ONLY (imported by tests/).  ``w`` is a dict of tensor name -> array, ``cfg`` the
parsed config.json."""
from __future__ import annotations

import numpy as np


def f64(a):
    return np.asarray(a, dtype=np.float64)


# ---- pointwise ---------------------------------------------------------------------------------
def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def relu_squared(z):
    return np.square(np.maximum(z, 0.0))


def over_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) along the last axis."""
    return x / np.sqrt(np.mean(np.square(x), axis=-1, keepdims=True) + eps)


def unit_vectors(x):
    return x / np.sqrt(np.sum(np.square(x), axis=-1, keepdims=True) + 1e-6)


#: what forward(rounding=...) applies to the inputs of matrix products and to stored keys and values
_rounding = None


def rounded(x):
    return f64(x) if _rounding is None else f64(_rounding(x)).reshape(np.shape(x))


def linear(h, weight):
    return rounded(h) @ f64(weight).T


# ---- short convolution -------------------------------------------------------------------------
def short_conv(x, taps, bias=None):
    """x [T, C]; taps [C, n], oldest first; nothing precedes token 0."""
    x, taps = f64(x), f64(taps)
    T, C = x.shape
    n = taps.shape[1]
    y = np.zeros((T, C))
    for t in range(T):
        for j in range(n):
            s = t - (n - 1 - j)
            if s >= 0:
                y[t] += taps[:, j] * x[s]
    if bias is not None:
        y = y + f64(bias)
    return y


# ---- recurrences -------------------------------------------------------------------------------
def delta_rule(q, k, v, beta, g, state=None):
    """q, k [T, H, K]; v [T, H, V]; beta [T, H]; g [T, H, K] (row decays).  -> outputs [T, H, V], state."""
    T, H, K = q.shape
    V = v.shape[-1]
    S = np.zeros((H, K, V)) if state is None else f64(state).copy()
    o = np.zeros((T, H, V))
    for t in range(T):
        for h in range(H):
            M = g[t, h][:, None] * S[h]
            u = beta[t, h] * (v[t, h] - M.T @ k[t, h])
            M = M + np.outer(k[t, h], u)
            S[h] = M
            o[t, h] = M.T @ q[t, h]
    return o, S


def state_space(x, B, C, dt, a_log, d_skip, state=None):
    """x [T, H, P]; B, C [T, H, N]; dt [T, H] (after softplus).  -> y [T, H, P], state [H, N, P]."""
    T, H, P = x.shape
    S = np.zeros((H, B.shape[-1], P)) if state is None else f64(state).copy()
    y = np.zeros((T, H, P))
    rate = np.exp(f64(a_log))
    for t in range(T):
        for h in range(H):
            S[h] = np.exp(-rate[h] * dt[t, h]) * S[h] + dt[t, h] * np.outer(B[t, h], x[t, h])
            y[t, h] = S[h].T @ C[t, h] + d_skip[h] * x[t, h]
    return y, S


# ---- attention ---------------------------------------------------------------------------------
def window_attention(q, k, v, scale, window):
    """q [T, H, K]; k [T, G, K]; v [T, G, V]; token i sees j with 0 <= i - j < window."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = np.zeros((T, H, v.shape[-1]))
    for i in range(T):
        lo = max(0, i - window + 1)
        for h in range(H):
            s = (k[lo:i + 1, h // per] @ q[i, h]) * scale
            p = np.exp(s - s.max())
            out[i, h] = (p / p.sum()) @ v[lo:i + 1, h // per]
    return out


# ---- mixers ------------------------------------------------------------------------------------
def _heads(x, n):
    return x.reshape(x.shape[0], n, -1)


def _delta_inputs(h, w, p, mix):
    qkv = {}
    for name in ("q", "k", "v"):
        qkv[name] = silu(short_conv(linear(h, w[f"{p}.{name}"]), w[f"{p}.{name}.conv"]))
    H, G, K = mix["heads"], mix["kv_heads"], mix["dim"]
    q = np.repeat(unit_vectors(_heads(qkv["q"], G)), H // G, axis=1) * K ** -0.5
    k = np.repeat(unit_vectors(_heads(qkv["k"], G)), H // G, axis=1)
    return q, k, _heads(qkv["v"], H), sigmoid(linear(h, w[f"{p}.b"]))


def mixer_delta(h, w, p, mix, eps):
    q, k, v, beta = _delta_inputs(h, w, p, mix)
    g = np.exp(-np.exp(f64(w[f"{p}.A_log"])) * softplus(linear(h, w[f"{p}.a"]) + f64(w[f"{p}.dt_bias"])))
    o, _ = delta_rule(q, k, v, beta, np.repeat(g[:, :, None], mix["dim"], axis=2))
    y = over_rms(o, eps) * f64(w[f"{p}.norm"]) * silu(_heads(linear(h, w[f"{p}.g"]), mix["heads"]))
    return linear(y.reshape(len(h), -1), w[f"{p}.o"])


def mixer_channel_delta(h, w, p, mix, eps):
    q, k, v, beta = _delta_inputs(h, w, p, mix)
    a = linear(linear(h, w[f"{p}.a1"]), w[f"{p}.a2"]) + f64(w[f"{p}.dt_bias"])
    g = np.exp(-np.exp(f64(w[f"{p}.A_log"]))[None, :, None] * _heads(softplus(a), mix["heads"]))
    o, _ = delta_rule(q, k, v, beta, g)
    gate = sigmoid(_heads(linear(linear(h, w[f"{p}.g1"]), w[f"{p}.g2"]), mix["heads"]))
    y = over_rms(o, eps) * f64(w[f"{p}.norm"]) * gate
    return linear(y.reshape(len(h), -1), w[f"{p}.o"])


def mixer_window(h, w, p, mix, eps):
    H, G = mix["heads"], mix["kv_heads"]
    q = over_rms(_heads(linear(h, w[f"{p}.q"]), H), eps) * f64(w[f"{p}.q.norm"])
    k = over_rms(_heads(linear(h, w[f"{p}.k"]), G), eps) * f64(w[f"{p}.k.norm"])
    v = _heads(linear(h, w[f"{p}.v"]), G)
    o = window_attention(q, rounded(k), rounded(v), mix["scale"], mix["mask"]["size"])
    return linear(o.reshape(len(h), -1), w[f"{p}.o"])


def mixer_state_space(h, w, p, mix, eps):
    H, P, N, G = mix["heads"], mix["vdim"], mix["state"], mix["groups"]
    inner = H * P
    z, xbc, dt = np.split(linear(h, w[f"{p}.in"]), [inner, 2 * inner + 2 * G * N], axis=1)
    xbc = silu(short_conv(xbc, w[f"{p}.conv"], w[f"{p}.conv.b"]))
    x, B, C = np.split(xbc, [inner, inner + G * N], axis=1)
    spread = lambda m: np.repeat(_heads(m, G), H // G, axis=1)
    y, _ = state_space(_heads(x, H), spread(B), spread(C), softplus(dt + f64(w[f"{p}.dt_bias"])),
                       w[f"{p}.A_log"], f64(w[f"{p}.D"]))
    y = y.reshape(len(h), -1) * silu(z)
    y = over_rms(_heads(y, mix["norm_groups"]), eps).reshape(len(h), -1) * f64(w[f"{p}.norm"])
    return linear(y, w[f"{p}.o"])


def mixer_parallel(h, w, p, mix, eps):
    return mix["left_scale"] * mixer_window(h, w, p + ".left", mix["left"], eps) + \
        mix["right_scale"] * mixer_state_space(h, w, p + ".right", mix["right"], eps)


MIXERS = {"delta": mixer_delta, "channel_delta": mixer_channel_delta, "parallel": mixer_parallel}


# ---- model -------------------------------------------------------------------------------------
def feed_forward(h, w, p):
    return linear(relu_squared(linear(h, w[f"{p}.up"])), w[f"{p}.down"])


def forward(cfg, w, tokens, want_layers=False, rounding=None):
    """Logits [T, vocab] of one sequence from position 0 (and the residual stream after every layer).
    rounding: applied where activations of lower precision enter matrix products or a cache."""
    global _rounding
    _rounding = rounding
    try:
        return _forward(cfg, w, tokens, want_layers)
    finally:
        _rounding = None


def _forward(cfg, w, tokens, want_layers):
    eps = cfg["norm"]["eps"]
    tokens = np.asarray(tokens)
    x = f64(w["embed"])[tokens] + f64(w["pos"])[:len(tokens)]
    history, after = [x], []
    for i, layer in enumerate(cfg["layers"]):
        h = over_rms(x, eps) * float(f64(w[f"l{i}.norm1"]).reshape(()))
        y = MIXERS[layer["type"]](h, w, f"l{i}.mix", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            y = y + feed_forward(h, w, f"l{i}.mlp")
        history.append(x + y)
        x = sum(float(c) * X for c, X in zip(f64(w[f"l{i}.dwa"]), history))
        after.append(x)
    logits = linear(over_rms(x, eps) * float(f64(w["final.norm"]).reshape(())), w["head"])
    return (logits, after) if want_layers else logits
