"""Small random Netinex models for the tests: configurations and bf16-representable weights.

A token's first TYPES embedding columns are large and name one of as many types of token, so that every norm
saturates there, and the routers read mostly those: which experts a token gets is then a matter of wide margins,
not of rounding.  The last norm turns these columns down again."""
import copy

import numpy as np

from nezavik_models import bf16

TYPES = 8


def moe(ff=40, experts=6, top=2):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def retention(heads=3, dim=24, vdim=40, dims=16, base=10000.0, decay=None, mlp=None):
    decay = decay or [round(1 - 2.0 ** -(2 + 2 * (h % 5)), 6) for h in range(heads)]
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay,
                                           "rot": {"base": base, "dims": dims}}, "mlp": mlp}


def attention(heads=4, kv=2, dim=32, dims=32, base=5000.0, size=30, scale=0.2, scaling=None, mlp=None):
    rot = {"base": base, "dims": dims}
    if scaling:
        rot["scaling"] = scaling
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": scale,
                                           "mask": {"size": size}, "rot": rot}, "mlp": mlp}


YARN = {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}


def config(layers, vocab=90, width=72, eps=1e-5, softcap=15.0):
    cfg = {"architecture": "Netinex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": copy.deepcopy(layers)}
    if softcap:
        cfg["logit_softcap"] = softcap
    return cfg


def weights(cfg, seed=0):
    rng = np.random.default_rng(seed)
    W, V = cfg["width"], cfg["vocab"]
    w = {}

    def lin(name, o, i, gain=1.0):
        w[name] = gain * rng.standard_normal((o, i)) / np.sqrt(i)

    def norm(name):
        w[name] = rng.uniform(0.6, 1.5, W)
        w[name + ".b"] = 0.2 * rng.standard_normal(W)
        w[name + ".alpha"] = np.array(rng.uniform(0.5, 1.1))

    types = TYPES if W >= 4 * TYPES else 0
    w["embed"] = rng.standard_normal((V, W))
    if types:
        w["embed"][:, :types] = 12.0 * np.eye(types)[rng.integers(0, types, V)] - 6.0
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix", layer["mixer"]
        norm(f"l{i}.norm1")
        H = m["heads"]
        G = m.get("kv_heads", H)
        lin(p + ".q", H * m["dim"], W)
        lin(p + ".k", G * m["dim"], W)
        if layer["type"] == "retention":
            lin(p + ".v", H * m["vdim"], W)
            lin(p + ".g", H * m["vdim"], W)
        else:
            w[p + ".q.norm"] = 1 + 0.3 * rng.standard_normal(H * m["dim"])
            w[p + ".k.norm"] = 1 + 0.3 * rng.standard_normal(G * m["dim"])
        lin(p + ".o", W, H * m["vdim"])
        w[p + ".o"][:types] *= 0.1
        if layer["mlp"]:
            norm(f"l{i}.norm2")
            w[f"l{i}.norm2"][:types], w[f"l{i}.norm2.b"][:types] = 1.0, 0.0
            p, e = f"l{i}.mlp", layer["mlp"]["router"]["experts"]
            ff = layer["mlp"]["expert"]["ff"]
            w[p + ".router"] = 0.1 * rng.standard_normal((e, W)) / np.sqrt(W)
            w[p + ".router.b"] = 0.5 * rng.standard_normal(e)
            if types:   # every type has its own order of the experts, 0.6 apart
                level = np.stack([rng.permutation(e) for _ in range(types)], axis=1) - 0.5 * (e - 1)
                table = 0.3 * level + 0.1 * (rng.random((e, types)) - 0.5)
                w[p + ".router"][:, :types] = table
                w[p + ".router.b"] = table.sum(axis=1)
            for x in range(e):
                lin(f"{p}.e{x}.gate", ff, W, 2.0)
                lin(f"{p}.e{x}.up", ff, W, 2.0)
                lin(f"{p}.e{x}.down", W, ff)
                w[f"{p}.e{x}.down"][:types] *= 0.1
    norm("final.norm")
    w["final.norm"][:types] *= 0.05
    w["final.norm.b"][:types] = 0.0
    return {k: bf16(v).reshape(np.shape(v)) for k, v in w.items()}
