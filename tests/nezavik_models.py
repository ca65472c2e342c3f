"""Small random Nezavik models for the tests: configurations, bf16-representable weights, and the
checkpoint folder the engine opens."""
import copy
import json
import os
import struct

import numpy as np


def bf16(a):
    u = np.ascontiguousarray(a, np.float32).view(np.uint32).astype(np.uint64)
    return ((u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000).astype(np.uint32).view(np.float32)


def delta(heads=2, kv=1, dim=24, vdim=40, conv=4, kind="delta", ff=96):
    return {"type": kind, "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def channel_delta(**kw):
    return delta(kind="channel_delta", **kw)


def parallel(heads=4, kv=2, dim=32, vdim=48, window=20, scale=0.2, ls=0.7, rs=1.1, s_heads=4, groups=2, state=40,
             s_vdim=24, conv=3, norm_groups=4, ff=96):
    return {"type": "parallel",
            "mixer": {"left": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale,
                               "mask": {"size": window}},
                      "left_scale": ls,
                      "right": {"heads": s_heads, "groups": groups, "state": state, "vdim": s_vdim, "conv": conv,
                                "norm_groups": norm_groups},
                      "right_scale": rs},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(layers, vocab=90, width=72, max_positions=512, eps=1e-5):
    return {"architecture": "Nezavik", "vocab": vocab, "width": width, "max_positions": max_positions,
            "norm": {"eps": eps}, "layers": copy.deepcopy(layers)}


def weights(cfg, seed=0, rank_a=12, rank_g=20):
    """Random weights whose recurrences remember: decays from about 0.5 to 0.999 per token."""
    rng = np.random.default_rng(seed)
    W, V = cfg["width"], cfg["vocab"]
    w = {}

    def lin(name, o, i):
        w[name] = rng.standard_normal((o, i)) / np.sqrt(i)

    def recurrence(p, heads, n_dt):
        w[p + ".A_log"] = rng.uniform(-5.0, -0.5, heads)
        w[p + ".dt_bias"] = rng.standard_normal(n_dt)

    w["embed"] = rng.standard_normal((V, W))
    w["pos"] = 0.3 * rng.standard_normal((cfg["max_positions"], W))
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix", layer["mixer"]
        w[f"l{i}.norm1"] = np.array(rng.uniform(0.7, 1.4))
        w[f"l{i}.dwa"] = 0.3 * rng.standard_normal(i + 2) + np.eye(i + 2)[-1]
        if layer["type"] == "parallel":
            a, s = m["left"], m["right"]
            lin(p + ".left.q", a["heads"] * a["dim"], W)
            lin(p + ".left.k", a["kv_heads"] * a["dim"], W)
            lin(p + ".left.v", a["kv_heads"] * a["vdim"], W)
            w[p + ".left.q.norm"] = 1 + 0.2 * rng.standard_normal(a["dim"])
            w[p + ".left.k.norm"] = 1 + 0.2 * rng.standard_normal(a["dim"])
            lin(p + ".left.o", W, a["heads"] * a["vdim"])
            inner, gn = s["heads"] * s["vdim"], s["groups"] * s["state"]
            lin(p + ".right.in", 2 * inner + 2 * gn + s["heads"], W)
            w[p + ".right.conv"] = 0.6 * rng.standard_normal((inner + 2 * gn, s["conv"]))
            w[p + ".right.conv.b"] = 0.3 * rng.standard_normal(inner + 2 * gn)
            recurrence(p + ".right", s["heads"], s["heads"])
            w[p + ".right.D"] = rng.standard_normal(s["heads"])
            w[p + ".right.norm"] = 1 + 0.2 * rng.standard_normal(inner)
            lin(p + ".right.o", W, inner)
        else:
            H, nk, nv = m["heads"], m["kv_heads"] * m["dim"], m["heads"] * m["vdim"]
            for name, n in (("q", nk), ("k", nk), ("v", nv)):
                lin(f"{p}.{name}", n, W)
                w[f"{p}.{name}.conv"] = 0.6 * rng.standard_normal((n, m["conv"]))
            lin(p + ".b", H, W)
            w[p + ".norm"] = 1 + 0.2 * rng.standard_normal(m["vdim"])
            lin(p + ".o", W, nv)
            if layer["type"] == "delta":
                recurrence(p, H, H)
                lin(p + ".a", H, W)
                lin(p + ".g", nv, W)
            else:
                recurrence(p, H, H * m["dim"])
                lin(p + ".a1", rank_a, W)
                lin(p + ".a2", H * m["dim"], rank_a)
                lin(p + ".g1", rank_g, W)
                lin(p + ".g2", nv, rank_g)
        if layer["mlp"]:
            lin(f"l{i}.mlp.up", layer["mlp"]["ff"], W)
            lin(f"l{i}.mlp.down", W, layer["mlp"]["ff"])
    w["final.norm"] = np.array(1.2)
    lin("head", V, W)
    return {k: bf16(v).reshape(np.shape(v)) for k, v in w.items()}


def save(path, cfg, w, dtype="BF16"):
    """config.json + model.safetensors in folder `path`."""
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    head, blobs, at = {"__metadata__": {"made": "by tests"}}, [], 0
    for name, t in w.items():
        b = (t.astype(np.float32).reshape(-1).view(np.uint32) >> 16).astype("<u2").tobytes() if dtype == "BF16" else \
            t.astype("<f4").tobytes()
        head[name] = {"dtype": dtype, "shape": list(t.shape), "data_offsets": [at, at + len(b)]}
        blobs.append(b)
        at += len(b)
    raw = json.dumps(head).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(raw)) + raw + b"".join(blobs))
    return path


def tokens(cfg, n, seed):
    return np.random.default_rng(seed + 1000).integers(0, cfg["vocab"], n).astype(np.int32)


def row_errors(got, want):
    """Per position: rms over the vocabulary of the difference (means taken off), over the logits' rms."""
    d = np.asarray(got, np.float64) - want
    d = d - d.mean(axis=-1, keepdims=True)
    centred = want - want.mean(axis=-1, keepdims=True)
    return np.sqrt((d ** 2).mean(axis=-1)) / np.sqrt((centred ** 2).mean())
