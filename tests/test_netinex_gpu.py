"""Netinex served by the engine, against the float64 restatement (oracle/netinex_oracle.py): each mechanism
alone, prompts against token-by-token decoding, portions, mixed batches, cache slots that are used again, chunk
edges, distant tokens, long decoding, unusual sizes, and generation through the scheduler.

fp32 (GPTOSS_ENGINE_PRECISE) is the sharp comparison; bf16 is what is served, and is compared with the
restatement whose matrix products and stored keys and values are bf16 as well.  Errors are per position,
relative to the rms of the logits."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from conftest import ROOT, load_pkg
import netinex_models as xm
import nezavik_models as nm
from engine_harness import feed, greedy, open_model, requests  # noqa: F401
from oracle import netinex_oracle as nx

pytestmark = pytest.mark.gpu

TOL = {True: 3e-5, False: 1.5e-2}      # keyed by `precise`
BOTH = pytest.mark.parametrize("precise", [True, False], ids=["fp32", "bf16"])


def restate(cfg, w, tok, precise):
    """Logits of every position in the engine's own precision; no router of the model may be near a tie."""
    margins = []
    want = nx.forward(cfg, w, tok, rnd=None if precise else nm.bf16, margins=margins)
    assert all(m.min() > 0.05 for m in margins)
    return want


def check(got, want, precise, factor=1.0):
    err = nm.row_errors(got, want)
    assert np.isfinite(got).all() and err.max() <= factor * TOL[precise], (err.max(), int(err.argmax()))


MIXED = [xm.retention(mlp=xm.moe()), xm.attention(mlp=xm.moe(experts=9, top=3), scaling=xm.YARN),
         xm.retention(heads=2, dim=40, vdim=16, dims=40, mlp=xm.moe(ff=70, experts=5, top=1)),
         xm.attention(heads=6, kv=3, dim=20, dims=12, size=47)]

MECHANISMS = {
    "retention": [xm.retention()],
    "retention_part_rotated": [xm.retention(heads=5, dim=33, vdim=65, dims=6, base=30.0)],
    "retention_rotated_in_fours": [xm.retention(heads=3, dim=36, vdim=68, dims=24, base=30.0)],
    "retention_rotated_in_twos": [xm.retention(heads=2, dim=28, vdim=20, dims=12)],
    "retention_fast_decay": [xm.retention(heads=4, decay=[0.0, 0.01, 0.25, 1.0])],
    "attention": [xm.attention()],
    "attention_scaled_part_rotated": [xm.attention(heads=6, kv=2, dim=48, dims=40, size=70, scaling=xm.YARN)],
    "attention_one_group": [xm.attention(heads=20, kv=1, dim=24, dims=24, size=50)],
    "experts": [xm.retention(mlp=xm.moe(experts=7, top=3))],
    "many_experts_per_token": [xm.attention(mlp=xm.moe(ff=24, experts=40, top=11))],
    "one_expert": [xm.attention(mlp=xm.moe(experts=1, top=1))],
    "every_expert": [xm.retention(mlp=xm.moe(experts=4, top=4))],
}


@BOTH
@pytest.mark.parametrize("name", MECHANISMS)
def test_each_mechanism_alone(open_model, name, precise):
    cfg = xm.config(MECHANISMS[name])
    w = xm.weights(cfg, 11)
    if "expert" in name:
        w["l0.mix.o"] = np.zeros_like(w["l0.mix.o"])
    tok = nm.tokens(cfg, 150, 3)
    want = restate(cfg, w, tok, precise)
    e = open_model(cfg, w, precise)
    check(feed(e, 0, tok), want, precise)
    check(feed(e, 1, tok, [70, 1]), want, precise)


@BOTH
def test_layers_without_softcap_or_feed_forward(open_model, precise):
    cfg = xm.config([xm.retention(), xm.attention()], softcap=None)
    w = xm.weights(cfg, 12)
    tok = nm.tokens(cfg, 60, 3)
    check(feed(open_model(cfg, w, precise), 0, tok, [40, 1]), restate(cfg, w, tok, precise), precise)


@BOTH
def test_first_tokens_of_a_sequence(open_model, precise):
    cfg = xm.config(MIXED[:2])
    w = xm.weights(cfg, 20)
    e = open_model(cfg, w, precise)
    for n in (1, 2, 3, 4, 5, 9):
        tok = nm.tokens(cfg, n, n)
        want = restate(cfg, w, tok, precise)
        check(feed(e, 1, tok), want, precise)
        check(feed(e, 1, tok, [1]), want, precise)


@BOTH
@pytest.mark.parametrize("cuts", [[1], [2], [3, 2], [5, 1, 1, 7], [64], [63, 1, 2], [130, 2, 1], [16], [17, 2, 31], [47, 46, 1],
                                  [8, 9], [65, 15], [10, 1, 1, 33]])
def test_portions_and_decoding_equal_the_whole_prompt(open_model, cuts, precise):
    cfg = xm.config(MIXED)
    w = xm.weights(cfg, 20)
    tok = nm.tokens(cfg, 170, 2)
    e = open_model(cfg, w, precise)
    want = restate(cfg, w, tok, precise)
    whole = feed(e, 0, tok)
    check(whole, want, precise)
    cut = feed(e, 1, tok, cuts)
    check(cut, want, precise)
    check(cut, whole.astype(np.float64), precise)


@BOTH
def test_batches_of_unequal_requests_equal_each_alone(open_model, precise):
    """Steps that mix decoding rows, short and long stretches and idle slots."""
    cfg = xm.config(MIXED)
    w = xm.weights(cfg, 26)
    e = open_model(cfg, w, precise, max_batch=5)
    toks = [nm.tokens(cfg, n, 40 + i) for i, n in enumerate((140, 33, 97, 2))]
    want = [restate(cfg, w, t, precise) for t in toks]
    plan = [[(0, 50)], [(0, 1), (1, 20)], [(2, 64), (0, 1), (1, 1)], [(1, 5), (3, 1)], [(0, 1), (1, 1), (2, 1), (3, 1)],
            [(2, 30), (0, 60)], [(0, 1), (2, 1)], [(1, 5), (0, 26), (2, 1)]]
    slots, at, got = [3, 0, 4, 1], [0] * 4, [[] for _ in toks]
    for step in plan:
        rows = [(i, at[i] + j) for i, n in step for j in range(n)]
        out = e.step_logits([toks[i][p] for i, p in rows], [slots[i] for i, _ in rows], [p for _, p in rows],
                            np.arange(len(rows)))
        for (i, p), lg in zip(rows, out):
            got[i].append(lg)
        for i, n in step:
            at[i] += n
    for i in range(4):
        assert at[i] == len(got[i]) and at[i] > 1
        check(np.array(got[i]), want[i][:len(got[i])], precise)


@BOTH
def test_slots_that_are_freed_and_used_again(open_model, precise):
    cfg = xm.config(MIXED)
    w = xm.weights(cfg, 24)
    e = open_model(cfg, w, precise, max_batch=2, max_seq=200)
    a, b = e.acquire_slot(), e.acquire_slot()
    lib = load_pkg("lib")
    with pytest.raises(lib.GptossError):
        e.acquire_slot()
    feed(e, a, nm.tokens(cfg, 120, 1), [50, 1])
    feed(e, b, nm.tokens(cfg, 70, 2))
    e.release_slot(a)
    assert e.acquire_slot() == a
    for n in (90, 3, 150):                     # shorter and longer than what the slot held before
        tok = nm.tokens(cfg, n, n)
        check(feed(e, a, tok, [40, 1, 2]), restate(cfg, w, tok, precise), precise)
    # the other slot went on undisturbed
    tok = np.concatenate([nm.tokens(cfg, 70, 2), nm.tokens(cfg, 9, 7)])
    check(feed(e, b, tok[70:], [1], start=70), restate(cfg, w, tok, precise)[70:], precise)


def test_a_sequence_cannot_continue_elsewhere(open_model):
    cfg = xm.config([xm.attention()])
    e = open_model(cfg, xm.weights(cfg, 1), max_seq=64)
    feed(e, 0, nm.tokens(cfg, 10, 1))
    lib = load_pkg("lib")
    for pos in (9, 11):
        with pytest.raises(lib.GptossError) as ei:
            e.step_logits([1], [0], [pos], [0])
        assert ei.value.code == 6
    with pytest.raises(lib.GptossError):       # beyond the engine's positions
        e.step_logits([1], [0], [64], [0])
    e.step_logits([1], [0], [10], [0])         # refused steps left the state alone


def _planted_chunk(size, dim=32, heads=4, kv=2):
    """A model of one attention layer in which one key stands out: token 1 (the marker) is the only one whose key
    points along the query of token 2 (the asker), and its key is also the value that moves the logits.  The
    directions lie in dimensions that are not rotated, so that no distance weakens them."""
    cfg = xm.config([xm.attention(heads=heads, kv=kv, dim=dim, dims=4, size=size, scale=1.0)], vocab=40, width=64)
    w = xm.weights(cfg, 77)
    rng = np.random.default_rng(2)
    p, W = "l0.mix", cfg["width"]
    emb = np.zeros((40, W))                    # columns: 0 the marker, 1 the asker, 2 everything else
    emb[:, 2], emb[1, :3], emb[2, :3] = 1.0, (1, 0, 0), (0, 1, 0)
    w["embed"] = nm.bf16(emb * 2 + 0.02 * rng.standard_normal((40, W)))
    q, k = np.zeros((heads * dim, W)), np.zeros((kv * dim, W))
    along, other = rng.standard_normal(dim), rng.standard_normal(dim)
    along[:4] = other[:4] = 0.0
    other -= along * (along @ other) / (along @ along)
    for h in range(heads):
        q[h * dim:(h + 1) * dim, :3] = np.stack([other, along, other], 1)
    for g in range(kv):
        k[g * dim:(g + 1) * dim, :3] = np.stack([along, other, other], 1)
    w[p + ".q"], w[p + ".k"] = nm.bf16(q), nm.bf16(k)
    w[p + ".q.norm"], w[p + ".k.norm"] = np.ones(heads * dim, np.float32), np.ones(kv * dim, np.float32)
    w["l0.norm1.b"] = np.zeros(W, np.float32)
    return cfg, w


@BOTH
@pytest.mark.parametrize("size", [1, 2, 31, 64, 65, 100])
def test_chunk_edges_in_prompts_and_in_decoding(open_model, size, precise):
    """A marker at the first position of the asker's chunk shows in its logits, at the last position of the
    chunk before it does not: with the asker first, second and last of its chunk, in a prompt, alone, and first
    or second of a portion."""
    cfg, w = _planted_chunk(size)
    e = open_model(cfg, w, precise, max_seq=320)
    base = nm.tokens(cfg, 320, 9) % 30 + 5
    for chunk in sorted({1, 128 // size, 160 // size + 1}):
        first = chunk * size
        for ask in sorted({first, first + 1, first + size - 1}):
            if ask >= first + size:
                continue
            seen = {}
            for name, at in (("inside", first), ("outside", first - 1)):
                tok = base[:ask + 1].copy()
                tok[ask] = 2
                if at != ask:
                    tok[at] = 1
                want = restate(cfg, w, tok, precise)
                seen[name] = want[ask]
                check(feed(e, 0, tok), want, precise)
                check(feed(e, 1, tok, [ask, 1]), want, precise)
                check(feed(e, 2, tok, [ask - 1, 2] if ask > 1 else [1]), want, precise)
            if ask > first:
                assert nm.row_errors(seen["inside"][None], seen["outside"][None])[0] > 5 * TOL[False]


@BOTH
def test_distant_tokens_reach_the_end(open_model, precise):
    """Heads that hardly decay: the first tokens still move the last logits hundreds of tokens later (in the
    restatement by far more than the tolerance), and the engine agrees."""
    cfg = xm.config([xm.retention(heads=2, decay=[1.0, 0.9999], dims=8, base=1e6), xm.attention(size=9),
                     xm.retention(heads=1, decay=[0.99999], dims=2)])
    w = xm.weights(cfg, 51)
    n = 600
    tok = nm.tokens(cfg, n, 4) % 10
    other = tok.copy()
    other[:60] = nm.tokens(cfg, 60, 5) % 60 + 30
    e = open_model(cfg, w, precise, max_seq=n)
    want, changed = restate(cfg, w, tok, precise), restate(cfg, w, other, precise)
    assert nm.row_errors(changed[-1:], want[-1:])[0] > 2 * TOL[False]
    check(feed(e, 0, tok, [256, 300, 1]), want, precise)
    check(feed(e, 1, other, [n]), changed, precise)


@BOTH
def test_long_decoding_past_the_ring(open_model, precise):
    """More positions than a pass or the ring holds: a prompt of several passes, then decoding."""
    cfg = xm.config([xm.attention(heads=2, kv=1, dim=8, dims=8, size=50, scaling=xm.YARN, mlp=xm.moe(ff=16, experts=3, top=1)),
                     xm.retention(heads=1, dim=8, vdim=8, dims=8)], vocab=33, width=32)
    w = xm.weights(cfg, 61)
    tok = nm.tokens(cfg, 2420, 6)
    want = restate(cfg, w, tok, precise)
    e = open_model(cfg, w, precise, max_batch=2, max_seq=2500)
    # among thousands of positions of a 32-wide model a few multiply a rounding many times over
    factor = 4.0
    check(feed(e, 0, tok, [2300, 1]), want, precise, factor)
    check(feed(e, 1, tok, [700, 1, 2, 900, 64]), want, precise, factor)
    check(feed(e, 1, tok, [3, 1100, 1, 1030, 64]), want, precise, factor)


SIZES = {
    "least": xm.config([xm.retention(heads=1, dim=2, vdim=1, dims=2, decay=[0.5], mlp=xm.moe(ff=1, experts=1, top=1)),
                        xm.attention(heads=1, kv=1, dim=2, dims=2, size=1, mlp=xm.moe(ff=1, experts=2, top=2))],
                       vocab=5, width=3),
    "odd": xm.config([xm.attention(heads=9, kv=3, dim=31, dims=22, size=33, mlp=xm.moe(ff=131, experts=7, top=5)),
                      xm.retention(heads=7, dim=50, vdim=27, dims=34, mlp=xm.moe(ff=33, experts=11, top=1)),
                      xm.retention(heads=5, dim=45, vdim=99, dims=44)], vocab=203, width=150),
    "large_heads": xm.config([xm.retention(heads=2, dim=256, vdim=300, dims=256),
                              xm.attention(heads=2, kv=1, dim=256, dims=128, size=70, scale=0.06),
                              xm.retention(heads=1, dim=160, vdim=128, dims=32, mlp=xm.moe(ff=256, experts=4, top=2))],
                             vocab=64, width=128),
    "keys_of_every_width": xm.config([xm.retention(heads=2, dim=d, vdim=v, dims=r)
                                      for d, v, r in ((64, 64, 64), (96, 32, 48), (128, 132, 128), (192, 48, 64), (224, 16, 224))],
                                     width=160),
    "many_heads": xm.config([xm.attention(heads=40, kv=2, dim=16, dims=16, size=24),
                             xm.retention(heads=24, dim=8, vdim=16, dims=4, mlp=xm.moe(experts=33, top=8))],
                            vocab=128, width=192, eps=1e-2, softcap=4.0),
    "attention_of_many_heads": xm.config([xm.attention(heads=h, kv=g, dim=64, dims=d, size=50, scale=0.1)
                                          for h, g, d in ((48, 16, 64), (64, 32, 32), (96, 48, 60))], width=40),
    "wide_heads": xm.config([xm.attention(heads=4, kv=4, dim=96, dims=96, size=60, scale=0.1),
                             xm.attention(heads=8, kv=1, dim=128, dims=64, size=90, scale=0.09, scaling=xm.YARN)],
                            width=256),
}


@BOTH
@pytest.mark.parametrize("name", SIZES)
def test_other_sizes(open_model, name, precise):
    cfg = SIZES[name]
    w = xm.weights(cfg, 71)
    tok = nm.tokens(cfg, 140, 8)
    margins = []
    want = nx.forward(cfg, w, tok, rnd=None if precise else nm.bf16, margins=margins)
    assert all(m.min() > 0.05 for m in margins)
    e = open_model(cfg, w, precise, max_batch=2, max_seq=140)
    factor = 6.0 if name == "least" else 1.0      # three-wide rows: little averaging of roundings
    check(feed(e, 0, tok), want, precise, factor)
    check(feed(e, 1, tok, [70, 1, 2, 13, 1]), want, precise, factor)


@BOTH
@pytest.mark.parametrize("scaling", [None, {"factor": 8.0, "original": 40, "fast": 4.0, "slow": 0.5},
                                     {"factor": 2.0, "original": 1, "fast": 9.0, "slow": 8.0},
                                     {"factor": 0.5, "original": 100000, "fast": 2.0, "slow": 1.0}],
                         ids=["plain", "ramp", "all_divided", "none_divided"])
def test_rotation_far_from_the_start(open_model, scaling, precise):
    """Keys hundreds of positions apart in one chunk, with every form of the frequencies."""
    cfg = xm.config([xm.attention(heads=2, kv=1, dim=24, dims=20, base=300.0, size=1000, scale=0.4, scaling=scaling)])
    w = xm.weights(cfg, 33)
    tok = nm.tokens(cfg, 420, 5)
    e = open_model(cfg, w, precise, max_seq=420)
    check(feed(e, 0, tok, [300, 1, 90, 1]), restate(cfg, w, tok, precise), precise)


@BOTH
def test_wide_rows_and_passes_of_thousands_of_rows(open_model, precise):
    """Sizes at which the products cut their sum over K into parts (few rows, many inputs) and run on the
    256-row tiles (2048 rows and more in a pass, several sequences; hundreds of rows per expert)."""
    cfg = xm.config([xm.retention(heads=4, dim=64, vdim=128, dims=64, mlp=xm.moe(ff=256, experts=4, top=2)),
                     xm.attention(heads=8, kv=2, dim=64, dims=64, size=300, scale=0.125, mlp=xm.moe(ff=300, experts=3, top=2))],
                    vocab=96, width=320)
    w = xm.weights(cfg, 73)
    lens = (800, 790, 810)
    toks = [nm.tokens(cfg, n, n) for n in lens]
    want = [restate(cfg, w, t, precise) for t in toks]
    e = open_model(cfg, w, precise, max_batch=3, max_seq=900)
    tok, slot, pos = (np.concatenate(x) for x in zip(*[(t[:-5], [i] * (len(t) - 5), np.arange(len(t) - 5))
                                                       for i, t in enumerate(toks)]))
    got = np.split(e.step_logits(tok, slot, pos, np.arange(len(tok))), np.cumsum([n - 5 for n in lens])[:-1])
    for i in range(3):
        check(got[i], want[i][:-5], precise)
    for k in range(5):      # decoding: three rows at a time
        at = [n - 5 + k for n in lens]
        lg = e.step_logits([t[p] for t, p in zip(toks, at)], [0, 1, 2], at, [0, 1, 2])
        for i in range(3):
            check(lg[i:i + 1], want[i][at[i]:at[i] + 1], precise)


def test_missing_and_misshapen_tensors_are_named(ops, tmp_path):
    cfg = xm.config([xm.retention(), xm.attention(mlp=xm.moe())])
    w = xm.weights(cfg, 3)
    lib = load_pkg("lib")
    for change in ("l0.mix.g", "l0.norm1.alpha", "l1.mix.q.norm", "l1.mlp.e3.up", "l1.mlp.router.b", "final.norm.b", "embed"):
        for bad in ({k: v for k, v in w.items() if k != change}, {**w, change: np.ones((3, 3), np.float32)}):
            with pytest.raises(lib.GptossError) as ei:
                load_pkg("engine").Engine.open(nm.save(str(tmp_path / "bad"), cfg, bad))
            assert change in str(ei.value)
    for path, value in ((("mixer", "decay"), [0.5]), (("mixer", "rot"), {"dims": 3, "base": 10.0}), (("type",), "other")):
        bad = json.loads(json.dumps(cfg))
        at = bad["layers"][0]
        for key in path[:-1]:
            at = at[key]
        at[path[-1]] = value
        with pytest.raises(lib.GptossError):
            load_pkg("engine").Engine.open(nm.save(str(tmp_path / "bad"), bad, w))


# ---- generation ----------------------------------------------------------------------------------
def test_greedy_generation_through_the_scheduler(open_model):
    """More requests than slots, prompts of unequal length, length limits per request: every request gets
    the ids it would get alone."""
    cfg = xm.config([xm.retention(mlp=xm.moe()), xm.attention(size=7, mlp=xm.moe()), xm.retention(heads=2)])
    w = xm.weights(cfg, 91)
    prompts, n_prompt, ids = requests(cfg)
    limit = n_prompt + 13
    e = open_model(cfg, w, True, max_batch=3, max_seq=64)
    out, n = e.generate(ids, int(limit.max()), n_prompt=n_prompt, max_len=limit)
    forward = lambda seq: nx.forward(cfg, w, seq)
    compared = 0
    for i, p in enumerate(prompts):
        got = [int(t) for t in out[i][:int(np.argmax(out[i] < 0))]]
        # the scheduler visits limit - 1 positions: the last id comes from position limit - 2
        want, margin = greedy(forward, p, int(limit[i]))
        assert len(got) == len(want) - 1 or len(got) == len(want)
        if margin > 1e-3:
            compared += 1
            assert got == want[:len(got)], i
    assert compared >= 4
    # the lock-step entry points and the prompt pass give the same ids
    b = open_model(cfg, w, True, max_batch=3, max_seq=64)
    three = np.stack([nm.tokens(cfg, 12, s) for s in (1, 2, 3)])
    nxt = b.prefill(three)
    a = [b.step(nxt, 12)]
    a.append(b.step_ragged(a[0], [13, 13, 13]))
    for i in range(3):
        want, margin = greedy(forward, three[i], 15)
        if margin > 1e-3:
            assert [int(nxt[i]), int(a[0][i]), int(a[1][i])] == want


def test_bf16_generation_matches_its_own_logits(open_model):
    """Without kept logits the classifier's fused arg-max picks the ids: they are the arg-max of the logits
    a second engine computes for the same sequences (vocabularies that are padded included)."""
    cfg = xm.config(MIXED, vocab=101)
    w = xm.weights(cfg, 92)
    prompts, n_prompt, ids = requests(cfg)
    e = open_model(cfg, w, False, max_batch=3, max_seq=80, keep_logits=False)
    out, _ = e.generate(ids, 60, n_prompt=n_prompt)
    ref = open_model(cfg, w, False, max_batch=3, max_seq=80)
    wrong = total = 0
    for i, p in enumerate(prompts):
        got = out[i][:int(np.argmax(out[i] < 0))]
        assert got.min() >= 0 and got.max() < 101
        seq = np.concatenate([p, got])
        lg = feed(ref, 0, seq, [len(p), 1])[len(p) - 1:-1]
        best = lg.max(axis=1) - lg[np.arange(len(got)), got]
        wrong += int((best > 0.02 * lg.std()).sum())     # an id that is not (nearly) the best
        total += len(got)
    assert wrong == 0 and total > 150


def test_command_line_generates_and_replays(open_model, tmp_path):
    cfg = xm.config([xm.retention(mlp=xm.moe()), xm.attention(size=6)])
    w = xm.weights(cfg, 93)
    e = open_model(cfg, w, True, max_batch=2, max_seq=40)
    prompts, n_prompt, ids = requests(cfg)
    out, _ = e.generate(ids[:3, :23], 23 + 9, n_prompt=n_prompt[:3], max_len=n_prompt[:3] + 8)
    cmd = [sys.executable, os.path.join(ROOT, "bin", "gptoss"), "generate", "--model", e.path, "--dtype", "float32",
           "--max-new", "8", "--batch", "2"]
    for p in prompts[:3]:
        cmd += ["--prompt", ",".join(map(str, p))]
    r = subprocess.run(cmd, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    got = [[int(t) for t in line.split()] for line in r.stdout.splitlines()]
    assert got == [[int(t) for t in row[:int(np.argmax(row < 0))]] for row in out]

    tok = nm.tokens(cfg, 30, 1)
    steps = [{"entries": [{"id": "a", "tokens": tok[:20].tolist(), "want": [19, 0]}], "end": []},
             {"entries": [{"id": "a", "tokens": tok[20:22].tolist(), "want": []}], "end": []},
             {"entries": [{"id": "a", "tokens": tok[22:].tolist(), "want": [7, 3]}], "end": ["a"]},
             {"entries": [{"id": "b", "tokens": tok[:12].tolist(), "want": [11]}], "end": ["b"]}]
    wanted = [19, 0], [], [29, 25], [11]
    lines = "".join(json.dumps({"step": i, **s}) + "\n" for i, s in enumerate(steps))
    for dtype, precise in (("float32", True), ("bfloat16", False)):
        r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", e.path, "--dtype", dtype, "--out",
                            str(tmp_path), "--max-tokens", "30"], input=lines, capture_output=True, text=True, timeout=100)
        assert r.returncode == 0, r.stderr[-2000:]
        assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
        want = restate(cfg, w, tok, precise)
        for i, places in enumerate(wanted):
            path = tmp_path / f"{i}.f32"
            assert path.exists() == bool(places)
            if places:
                check(np.fromfile(path, "<f4").reshape(len(places), cfg["vocab"]), want[places], precise)
