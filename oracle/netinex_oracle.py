"""Plain float64 numpy restatement of the Netinex decoder: one function per mechanism, a token loop for the
recurrence, dense masked softmax for the attention, no caches and no batching.  Shares no code with the
product.

TEST INFRASTRUCTURE ONLY (imported by tests/).  ``w`` is a dict of tensor name -> array, ``cfg`` the
parsed config.json.  ``rnd`` is applied where activations of lower precision enter matrix products or a
cache (identity by default)."""
from __future__ import annotations

import math

import numpy as np


def f64(a):
    return np.asarray(a, dtype=np.float64)


def exact(x):
    return x


# ---- pointwise and norms -----------------------------------------------------------------------
def silu(z):
    e = np.exp(-np.abs(z))
    return z * np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def over_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) along the last axis."""
    return x / np.sqrt(np.mean(np.square(x), axis=-1, keepdims=True) + eps)


def tanh_norm(x, weight, bias, alpha):
    return np.tanh(float(f64(alpha).reshape(())) * x) * f64(weight) + f64(bias)


def softcap(z, cap):
    return cap * np.tanh(z / cap)


def linear(h, weight, rnd=exact):
    return f64(rnd(h)) @ f64(weight).T


# ---- rotation ----------------------------------------------------------------------------------
def frequencies(rot):
    """Angles per position, [dims / 2], and what cos and sin are multiplied by."""
    n, base = rot["dims"], float(rot["base"])
    f = [base ** (-2.0 * i / n) for i in range(n // 2)]
    s = rot.get("scaling")
    if s is None:
        return np.array(f), 1.0

    def place(turns):
        return n * math.log(s["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(place(s["fast"])), 0), min(math.ceil(place(s["slow"])), n - 1)
    for i in range(n // 2):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        f[i] = f[i] / s["factor"] * ramp + f[i] * (1 - ramp)
    return np.array(f), 0.1 * math.log(s["factor"]) + 1.0


def rotate(x, positions, rot, interleaved):
    """x [T, heads, dim]: the first rot.dims of every head; pairs (2i, 2i + 1), or (i, i + dims / 2)."""
    f, gain = frequencies(rot)
    x, half = f64(x), rot["dims"] // 2
    out = x.copy()
    for i in range(half):
        a, b = (2 * i, 2 * i + 1) if interleaved else (i, i + half)
        angle = np.asarray(positions)[:, None] * f[i]
        c, s = gain * np.cos(angle), gain * np.sin(angle)
        out[:, :, a], out[:, :, b] = x[:, :, a] * c - x[:, :, b] * s, x[:, :, b] * c + x[:, :, a] * s
    return out


# ---- mixers ------------------------------------------------------------------------------------
def retention(q, k, v, decay, state=None):
    """q, k [T, H, K]; v [T, H, V]; decay [H].  -> outputs [T, H, V], state [H, K, V]."""
    T, H, K = q.shape
    S = np.zeros((H, K, v.shape[-1])) if state is None else f64(state).copy()
    d = f64(decay)[:, None, None]
    o = np.zeros(v.shape)
    for t in range(T):
        S = d * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hkv,hk->hv", S, q[t])
    return o, S


def chunk_attention(q, k, v, scale, size):
    """q [T, H, K]; k [T, G, K]; v [T, G, V]; token i sees j <= i of its own chunk of `size` positions."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    seen = (j <= i) & (i // size == j // size)
    out = np.zeros((T, H, v.shape[-1]))
    for h in range(H):
        s = np.where(seen, q[:, h] @ k[:, h // per].T * scale, -np.inf)
        p = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, h] = p / p.sum(axis=1, keepdims=True) @ v[:, h // per]
    return out


def _heads(x, n):
    return x.reshape(x.shape[0], n, -1)


def mixer_retention(h, w, p, mix, eps, rnd=exact):
    H, at = mix["heads"], np.arange(len(h))
    q = rotate(_heads(linear(h, w[f"{p}.q"], rnd), H), at, mix["rot"], False)
    k = rotate(_heads(linear(h, w[f"{p}.k"], rnd), H), at, mix["rot"], False) * mix["dim"] ** -0.5
    o, _ = retention(q, k, _heads(linear(h, w[f"{p}.v"], rnd), H), mix["decay"])
    y = over_rms(o, eps).reshape(len(h), -1) * silu(linear(h, w[f"{p}.g"], rnd))
    return linear(y, w[f"{p}.o"], rnd)


def mixer_attention(h, w, p, mix, eps, rnd=exact):
    H, G, at = mix["heads"], mix["kv_heads"], np.arange(len(h))
    q, k = linear(h, w[f"{p}.q"], rnd), linear(h, w[f"{p}.k"], rnd)
    v = _heads(k, G)
    q = rotate(_heads(over_rms(q, eps) * f64(w[f"{p}.q.norm"]), H), at, mix["rot"], True)
    k = rotate(_heads(over_rms(k, eps) * f64(w[f"{p}.k.norm"]), G), at, mix["rot"], True)
    o = chunk_attention(q, f64(rnd(k)), f64(rnd(v)), mix["scale"], mix["mask"]["size"])
    return linear(o.reshape(len(h), -1), w[f"{p}.o"], rnd)


MIXERS = {"retention": mixer_retention, "attention": mixer_attention}


# ---- feed-forward ------------------------------------------------------------------------------
def route(z, top):
    """Logits [T, E] -> chosen experts [T, top] and their weights (softmax over the chosen logits)."""
    ids = np.argsort(-z, axis=1, kind="stable")[:, :top]
    picked = np.take_along_axis(z, ids, axis=1)
    e = np.exp(picked - picked.max(axis=1, keepdims=True))
    return ids, e / e.sum(axis=1, keepdims=True)


def margin(z, top):
    """Distance of the last chosen logit from the first one that is not, per token."""
    order = -np.sort(-z, axis=1)
    return order[:, top - 1] - order[:, top] if top < z.shape[1] else np.full(len(z), np.inf)


def feed_forward(h, w, p, mlp, rnd=exact, margins=None):
    z = linear(h, w[f"{p}.router"], rnd) + f64(w[f"{p}.router.b"])
    ids, share = route(z, mlp["router"]["top"])
    if margins is not None:
        margins.append(margin(z, mlp["router"]["top"]))
    y = np.zeros(h.shape)
    for t in range(len(h)):
        x = h[t:t + 1]
        for e, s in zip(ids[t], share[t]):
            a = silu(linear(x, w[f"{p}.e{e}.gate"], rnd)) * linear(x, w[f"{p}.e{e}.up"], rnd)
            y[t] += s * linear(a, w[f"{p}.e{e}.down"], rnd)[0]
    return y


# ---- model -------------------------------------------------------------------------------------
def _norm(x, w, name):
    return tanh_norm(x, w[name], w[name + ".b"], w[name + ".alpha"])


def forward(cfg, w, tokens, want_layers=False, rnd=None, margins=None):
    """Logits [T, vocab] of one sequence from position 0 (and the residual stream after every layer).
    margins: a list that receives every router's margins."""
    eps = cfg["norm"]["eps"]
    rounding = exact if rnd is None else rnd
    rnd = lambda x: f64(rounding(x)).reshape(np.shape(x))
    x, after = f64(w["embed"])[np.asarray(tokens)], []
    for i, layer in enumerate(cfg["layers"]):
        x = x + MIXERS[layer["type"]](_norm(x, w, f"l{i}.norm1"), w, f"l{i}.mix", layer["mixer"], eps, rnd)
        if layer.get("mlp") is not None:
            x = x + feed_forward(_norm(x, w, f"l{i}.norm2"), w, f"l{i}.mlp", layer["mlp"], rnd, margins)
        after.append(x)
    logits = linear(_norm(x, w, "final.norm"), w["embed"], rnd)
    if cfg.get("logit_softcap"):
        logits = softcap(logits, cfg["logit_softcap"])
    return (logits, after) if want_layers else logits
