"""Nezavik served by the engine, against the float64 restatement (oracle/nezavik_oracle.py): each
mechanism alone, prompts against token-by-token decoding, portions, mixed batches, cache slots that are
used again, window edges, long decoding, unusual sizes, and generation through the scheduler.

fp32 (GPTOSS_ENGINE_PRECISE) is the sharp comparison; bf16 is what is served, and is compared with the
restatement whose matrix products take bf16 inputs as well (how far rounding carries a small random model
depends on its weights: the two agree far more closely than either does with the exact one).  Errors are
per position, relative to the rms of the logits."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from conftest import ROOT, load_pkg
import nezavik_models as nm
from engine_harness import feed, greedy, open_model, requests  # noqa: F401
from oracle import nezavik_oracle as nz

pytestmark = pytest.mark.gpu

TOL = {True: 2e-5, False: 3e-2}      # keyed by `precise`
STAGED_TOL = 1e-2                    # bf16 against the restatement with bf16 inputs
BOTH = pytest.mark.parametrize("precise", [True, False], ids=["fp32", "bf16"])


def check(got, want, precise, factor=1.0):
    err = nm.row_errors(got, want)
    assert np.isfinite(got).all() and err.max() <= factor * TOL[precise], (err.max(), int(err.argmax()))


def check_model(e, slot, cfg, w, tok, precise, cuts=None, factor=1.0):
    """Every position of one sequence against the restatement in the engine's own precision."""
    got = feed(e, slot, tok, cuts)
    if precise:
        check(got, nz.forward(cfg, w, tok), True, factor)
    else:
        check(got, nz.forward(cfg, w, tok, rounding=nm.bf16), False, factor * STAGED_TOL / TOL[False])


MIXED = [nm.delta(heads=4, kv=2), nm.parallel(), nm.channel_delta(heads=3, kv=3, dim=40, vdim=16, conv=2),
         nm.parallel(window=37, heads=6, kv=2, ff=None)]

MECHANISMS = {
    "delta": [nm.delta(ff=None)],
    "delta_grouped": [nm.delta(heads=6, kv=2, dim=33, vdim=65, ff=None)],
    "channel_delta": [nm.channel_delta(ff=None)],
    "channel_delta_grouped": [nm.channel_delta(heads=4, kv=2, dim=64, vdim=72, conv=5, ff=None)],
    "window": [nm.parallel(rs=0.0, ff=None)],
    "state_space": [nm.parallel(ls=0.0, ff=None)],
    "parallel": [nm.parallel(ff=None)],
    "feed_forward": [nm.delta()],
    "depth_average": [nm.delta(ff=None)] * 4,
}


@BOTH
@pytest.mark.parametrize("name", MECHANISMS)
def test_each_mechanism_alone(open_model, name, precise):
    cfg = nm.config(MECHANISMS[name])
    w = nm.weights(cfg, 11)
    if name == "feed_forward":
        w["l0.mix.o"] = np.zeros_like(w["l0.mix.o"])
    tok = nm.tokens(cfg, 150, 3)
    e = open_model(cfg, w, precise)
    check_model(e, 0, cfg, w, tok, precise)
    check_model(e, 1, cfg, w, tok, precise, [70, 1])


@BOTH
def test_first_tokens_of_a_sequence(open_model, precise):
    """Convolutions that reach past token 0: lengths below, at and above every number of taps, in one step
    and token by token."""
    cfg = nm.config([nm.delta(conv=5), nm.parallel(conv=4), nm.channel_delta(conv=2)])
    w = nm.weights(cfg, 5)
    e = open_model(cfg, w, precise)
    for n in (1, 2, 3, 4, 5, 6, 9):
        tok = nm.tokens(cfg, n, n)
        want = nz.forward(cfg, w, tok)
        check(feed(e, 1, tok), want, precise)
        check(feed(e, 1, tok, [1]), want, precise)


@BOTH
@pytest.mark.parametrize("cuts", [[1], [2], [3, 2], [5, 1, 1, 7], [64], [63, 1, 2], [130, 2, 1], [16], [17, 2, 31]])
def test_portions_and_decoding_equal_the_whole_prompt(open_model, cuts, precise):
    cfg = nm.config(MIXED)
    w = nm.weights(cfg, 21)
    tok = nm.tokens(cfg, 170, 2)
    e = open_model(cfg, w, precise)
    want = nz.forward(cfg, w, tok)
    whole = feed(e, 0, tok)
    check(whole, want, precise)
    cut = feed(e, 1, tok, cuts)
    check(cut, want, precise)
    check(cut, whole.astype(np.float64), precise)


@BOTH
def test_batches_of_unequal_requests_equal_each_alone(open_model, precise):
    """Steps that mix decoding rows, short and long stretches and idle slots."""
    cfg = nm.config(MIXED)
    w = nm.weights(cfg, 31)
    e = open_model(cfg, w, precise, max_batch=5)
    toks = [nm.tokens(cfg, n, 40 + i) for i, n in enumerate((140, 33, 97, 2))]
    want = [nz.forward(cfg, w, t) for t in toks]
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
    cfg = nm.config(MIXED)
    w = nm.weights(cfg, 41)
    e = open_model(cfg, w, precise, max_batch=2)
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
        check(feed(e, a, tok, [40, 1, 2]), nz.forward(cfg, w, tok), precise)
    # the other slot went on undisturbed
    tok = np.concatenate([nm.tokens(cfg, 70, 2), nm.tokens(cfg, 9, 7)])
    check(feed(e, b, tok[70:], [1], start=70), nz.forward(cfg, w, tok)[70:], precise)


def test_a_sequence_cannot_continue_elsewhere(open_model):
    cfg = nm.config([nm.delta()])
    e = open_model(cfg, nm.weights(cfg, 1))
    feed(e, 0, nm.tokens(cfg, 10, 1))
    lib = load_pkg("lib")
    for pos in (9, 11):
        with pytest.raises(lib.GptossError) as ei:
            e.step_logits([1], [0], [pos], [0])
        assert ei.value.code == 6
    with pytest.raises(lib.GptossError):       # a slot twice in one step
        e.step_logits([1, 2, 3], [0, 1, 0], [10, 0, 11], [0])
    with pytest.raises(lib.GptossError):       # beyond the engine's positions
        e.step_logits([1], [0], [cfg["max_positions"]], [0])
    e.step_logits([1], [0], [10], [0])         # refused steps left the state alone


def _planted_window(window, dim=32, vdim=16, heads=4, kv=2):
    """A model whose only mechanism is the window attention, in which one key stands out: token 1 (the
    marker) is the only one whose key points along the query of token 2 (the asker); its value moves the
    logits.  Without the marker in sight the asker averages values that are all alike."""
    cfg = nm.config([nm.parallel(heads=heads, kv=kv, dim=dim, vdim=vdim, window=window, scale=1.0, ls=4.0, rs=0.0, ff=None)],
                    vocab=40, width=64)
    w = nm.weights(cfg, 77)
    p = "l0.mix.left"
    W = cfg["width"]
    w["pos"] = np.zeros_like(w["pos"])
    # directions of the embedding: 0 marks the marker, 1 the asker, 2 everything else
    emb = np.zeros((40, W))
    emb[:, 2] = 1.0
    emb[1] = np.eye(W)[0]
    emb[2] = np.eye(W)[1]
    w["embed"] = nm.bf16(emb * 2 + 0.01 * np.random.default_rng(1).standard_normal((40, W)))
    rng = np.random.default_rng(2)
    q, k, v = np.zeros((heads * dim, W)), np.zeros((kv * dim, W)), 0.02 * rng.standard_normal((kv * vdim, W))
    along, other = rng.standard_normal(dim), rng.standard_normal(dim)
    other -= along * (along @ other) / (along @ along)
    for h in range(heads):
        q[h * dim:(h + 1) * dim, :3] = np.stack([other, along, other], 1)
    for g in range(kv):
        k[g * dim:(g + 1) * dim, :3] = np.stack([along, other, other], 1)
    v[:, 0] = rng.standard_normal(kv * vdim)
    for name, m in (("q", q), ("k", k), ("v", v)):
        w[f"{p}.{name}"] = nm.bf16(m)
    w[p + ".q.norm"] = w[p + ".k.norm"] = np.ones(dim, np.float32)
    w["l0.dwa"] = np.array([0.25, 1.0], np.float32)
    return cfg, w


@BOTH
@pytest.mark.parametrize("window", [1, 2, 31, 64, 65, 100])
def test_window_edges_in_prompts_and_in_decoding(open_model, window, precise):
    """The marker just inside the asker's window shows in its logits, one token further away it does not:
    at places around the borders of the 64-slot blocks, with the asker in a prompt, alone, and first or
    second of a portion."""
    cfg, w = _planted_window(window)
    e = open_model(cfg, w, precise)
    base = nm.tokens(cfg, 260, 9) % 30 + 5
    for ask in (window + 3, 127, 128, 129, 191, 259):
        far = {}
        for name, gap in (("inside", window - 1), ("outside", window)):
            tok = base[:ask + 1].copy()
            tok[ask] = 2
            if gap:
                tok[ask - gap] = 1
            want = nz.forward(cfg, w, tok)
            far[name] = want[ask]
            check(feed(e, 0, tok), want, precise)
            check(feed(e, 1, tok, [ask, 1]), want, precise)
            check(feed(e, 2, tok, [ask - 1, 2]), want, precise)
        if window > 1:
            change = nm.row_errors(far["inside"][None], far["outside"][None])[0]
            assert change > 5 * TOL[False], change


@BOTH
def test_distant_tokens_reach_the_end(open_model, precise):
    """Heads that hardly decay: the first tokens still move the last logits hundreds of tokens later (in
    the restatement by far more than the tolerance), and the engine agrees."""
    cfg = nm.config([nm.delta(heads=2, kv=2, conv=3), nm.parallel(window=9), nm.channel_delta(conv=2)], max_positions=700)
    w = nm.weights(cfg, 51)
    for i, p in ((0, "l0.mix"), (1, "l1.mix.right"), (2, "l2.mix")):
        w[p + ".A_log"] = np.full_like(w[p + ".A_log"], -9.0)
        if i != 1:
            w[p + ".b"] = np.zeros_like(w[p + ".b"])       # write strength 1/2: little is overwritten per token
    n = 600
    tok = nm.tokens(cfg, n, 4) % 10
    other = tok.copy()
    other[:60] = nm.tokens(cfg, 60, 5) % 60 + 30
    e = open_model(cfg, w, precise)
    want, changed = nz.forward(cfg, w, tok), nz.forward(cfg, w, other)
    assert nm.row_errors(changed[-1:], want[-1:])[0] > 2 * TOL[False]
    check(feed(e, 0, tok, [256, 300, 1]), want, precise)
    check(feed(e, 1, other, [n]), changed, precise)


@BOTH
def test_long_decoding_past_the_ring(open_model, precise):
    """More positions than a pass or the window ring holds: a prompt of several passes, then decoding."""
    cfg = nm.config([nm.parallel(heads=2, kv=1, dim=8, vdim=8, window=50, s_heads=2, groups=1, state=8, s_vdim=8,
                                 norm_groups=2, ff=16), nm.delta(heads=1, kv=1, dim=8, vdim=8, ff=None)],
                    vocab=33, width=32, max_positions=2500)
    w = nm.weights(cfg, 61)
    tok = nm.tokens(cfg, 2420, 6)
    e = open_model(cfg, w, precise, max_batch=2)
    # among thousands of positions of a 32-wide model a few multiply a rounding many times over
    factor = 1.0 if precise else 5.0
    check_model(e, 0, cfg, w, tok, precise, [2300, 1], factor)
    check_model(e, 1, cfg, w, tok, precise, [700, 1, 2, 900, 64], factor)


SIZES = {
    "ones": (nm.config([nm.delta(heads=1, kv=1, dim=1, vdim=1, conv=1, ff=1),
                        nm.parallel(heads=1, kv=1, dim=1, vdim=1, window=1, s_heads=1, groups=1, state=1, s_vdim=1, conv=1,
                                    norm_groups=1, ff=1),
                        nm.channel_delta(heads=1, kv=1, dim=1, vdim=1, conv=1, ff=3)], vocab=5, width=3), 1, 1),
    "odd": (nm.config([nm.parallel(heads=9, kv=3, dim=31, vdim=45, window=33, s_heads=6, groups=3, state=35, s_vdim=17,
                                   conv=6, norm_groups=2, ff=131),
                       nm.channel_delta(heads=6, kv=2, dim=50, vdim=27, conv=3, ff=70),
                       nm.delta(heads=5, kv=5, dim=45, vdim=99, conv=7, ff=33)], vocab=203, width=150), 7, 33),
    "large_heads": (nm.config([nm.parallel(heads=2, kv=1, dim=256, vdim=130, window=70, s_heads=2, groups=2, state=256,
                                           s_vdim=128, norm_groups=1),
                               nm.delta(heads=2, kv=1, dim=256, vdim=192),
                               nm.channel_delta(heads=1, kv=1, dim=160, vdim=256)], vocab=64, width=128), 64, 40),
    "many_heads": (nm.config([nm.parallel(heads=40, kv=2, dim=16, vdim=16, window=24, s_heads=20, groups=1, state=16,
                                          s_vdim=8, norm_groups=20), nm.delta(heads=24, kv=3, dim=8, vdim=8)],
                             vocab=128, width=192, eps=1e-2), 16, 16),
    "wide_heads": (nm.config([nm.parallel(heads=4, kv=4, dim=96, vdim=128, window=60, norm_groups=2),
                              nm.parallel(heads=8, kv=1, dim=128, vdim=96, window=90, norm_groups=1)], width=256), 8, 8),
}


@BOTH
@pytest.mark.parametrize("name", SIZES)
def test_other_sizes(open_model, name, precise):
    cfg, ra, rg = SIZES[name]
    w = nm.weights(cfg, 71, ra, rg)
    tok = nm.tokens(cfg, 140, 8)
    e = open_model(cfg, w, precise, max_batch=2)
    factor = 4.0 if name == "ones" else 1.0      # three-wide rows: little averaging of roundings
    check_model(e, 0, cfg, w, tok, precise, factor=factor)
    check_model(e, 1, cfg, w, tok, precise, [70, 1, 2, 13, 1], factor)


@BOTH
def test_wide_rows_and_passes_of_thousands_of_rows(open_model, precise):
    """Sizes at which the products cut their sum over K into parts (few rows, many inputs) and run on the
    256-row tiles (2048 rows and more in a pass, several sequences)."""
    cfg = nm.config([nm.channel_delta(heads=2, kv=1, dim=32, vdim=128, ff=1400),
                     nm.parallel(heads=2, kv=1, dim=64, vdim=64, window=100, s_heads=1, groups=1, state=64, s_vdim=64,
                                 norm_groups=1, ff=900)], vocab=96, width=320, max_positions=900)
    w = nm.weights(cfg, 73, 40, 60)
    lens = (800, 790, 810)
    toks = [nm.tokens(cfg, n, n) for n in lens]
    rounding = None if precise else nm.bf16
    want = [nz.forward(cfg, w, t, rounding=rounding) for t in toks]
    e = open_model(cfg, w, precise, max_batch=3)
    tok, slot, pos = (np.concatenate(x) for x in zip(*[(t[:-5], [i] * (len(t) - 5), np.arange(len(t) - 5))
                                                       for i, t in enumerate(toks)]))
    got = np.split(e.step_logits(tok, slot, pos, np.arange(len(tok))), np.cumsum([n - 5 for n in lens])[:-1])
    for i in range(3):
        check(got[i], want[i][:-5], precise, 1.0 if precise else STAGED_TOL / TOL[False])
    for k in range(5):      # decoding: three rows at a time
        at = [n - 5 + k for n in lens]
        lg = e.step_logits([t[p] for t, p in zip(toks, at)], [0, 1, 2], at, [0, 1, 2])
        for i in range(3):
            check(lg[i:i + 1], want[i][at[i]:at[i] + 1], precise, 1.0 if precise else STAGED_TOL / TOL[False])


def test_fp32_checkpoints_load(open_model, tmp_path):
    cfg = nm.config([nm.delta()])
    w = nm.weights(cfg, 3)
    path = nm.save(str(tmp_path / "f32"), cfg, w, dtype="F32")
    e = load_pkg("engine").Engine.open(path, precise=True)
    tok = nm.tokens(cfg, 20, 1)
    check(feed(e, 0, tok), nz.forward(cfg, w, tok), True)
    e.close()


def test_missing_and_misshapen_tensors_are_named(open_model, tmp_path):
    cfg = nm.config([nm.delta()])
    w = nm.weights(cfg, 3)
    lib = load_pkg("lib")
    for change in ("l0.mix.k.conv", "head", "l0.dwa"):
        for bad in ({k: v for k, v in w.items() if k != change}, {**w, change: np.ones((3, 3), np.float32)}):
            with pytest.raises(lib.GptossError) as ei:
                load_pkg("engine").Engine.open(nm.save(str(tmp_path / "bad"), cfg, bad))
            assert change in str(ei.value)


# ---- generation ----------------------------------------------------------------------------------
def _greedy(cfg, w, prompt, total):
    return greedy(lambda seq: nz.forward(cfg, w, seq), prompt, total)


def test_greedy_generation_through_the_scheduler(open_model):
    """More requests than slots, prompts of unequal length, length limits per request: every request gets
    the ids it would get alone."""
    cfg = nm.config([nm.delta(heads=2), nm.parallel(window=7), nm.channel_delta()])
    w = nm.weights(cfg, 91)
    prompts, n_prompt, ids = requests(cfg)
    limit = n_prompt + 13
    e = open_model(cfg, w, True, max_batch=3, max_seq=64)
    out, n = e.generate(ids, int(limit.max()), n_prompt=n_prompt, max_len=limit)
    compared = 0
    for i, p in enumerate(prompts):
        got = [int(t) for t in out[i][:int(np.argmax(out[i] < 0))]]
        # the scheduler visits limit - 1 positions: the last id comes from position limit - 2
        want, margin = _greedy(cfg, w, p, int(limit[i]))
        assert len(got) == len(want) - 1 or len(got) == len(want)
        if margin > 1e-3:
            compared += 1
            assert got == want[:len(got)], i
    assert compared >= 5
    # the lock-step entry points and the prompt pass give the same ids
    b = open_model(cfg, w, True, max_batch=3, max_seq=64)
    three = np.stack([nm.tokens(cfg, 12, s) for s in (1, 2, 3)])
    nxt = b.prefill(three)
    a = [b.step(nxt, 12)]
    a.append(b.step_ragged(a[0], [13, 13, 13]))
    for i in range(3):
        want, margin = _greedy(cfg, w, three[i], 15)
        if margin > 1e-3:
            assert [int(nxt[i]), int(a[0][i]), int(a[1][i])] == want


def test_bf16_generation_matches_its_own_logits(open_model):
    """Without kept logits the classifier's fused arg-max picks the ids: they are the arg-max of the logits
    a second engine computes for the same sequences (vocabularies that are padded included)."""
    cfg = nm.config(MIXED, vocab=101)
    w = nm.weights(cfg, 92)
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
    cfg = nm.config([nm.delta(), nm.parallel(window=6)])
    w = nm.weights(cfg, 93)
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

    toks = {"a": nm.tokens(cfg, 30, 1), "b": nm.tokens(cfg, 12, 2)}
    steps = [{"entries": [{"id": "a", "tokens": toks["a"][:20].tolist(), "want": [0, 19]}], "end": []},
             {"entries": [{"id": "b", "tokens": toks["b"].tolist(), "want": []},
                          {"id": "a", "tokens": toks["a"][20:22].tolist(), "want": [1]}], "end": ["b"]},
             {"entries": [{"id": "a", "tokens": toks["a"][22:].tolist(), "want": [7, 3]}], "end": ["a"]},
             {"entries": [{"id": "c", "tokens": toks["b"].tolist(), "want": [11]}], "end": ["c"]}]
    wanted = [("a", 0), ("a", 19)], [("a", 21)], [("a", 29), ("a", 25)], [("b", 11)]
    lines = "".join(json.dumps({"step": i, **s}) + "\n" for i, s in enumerate(steps))
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", e.path, "--dtype", "float32", "--out",
                        str(tmp_path), "--max-tokens", "64"], input=lines, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    want = {n: nz.forward(cfg, w, t) for n, t in toks.items()}
    for i, places in enumerate(wanted):
        lg = np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(len(places), cfg["vocab"])
        check(lg, np.stack([want[n][p] for n, p in places]), True)
