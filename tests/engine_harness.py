"""What the tests of the model classes behind the engine share: opening a saved model, feeding one sequence in
portions, greedy ids of a restatement, a set of unequal requests."""
import numpy as np
import pytest

from conftest import load_pkg
import nezavik_models as nm


@pytest.fixture
def open_model(ops, tmp_path):
    engines = []

    def make(cfg, w, precise=True, max_batch=4, max_seq=0, **kw):
        path = nm.save(str(tmp_path / f"m{len(engines)}"), cfg, w)
        e = load_pkg("engine").Engine.open(path, max_batch=max_batch, max_seq=max_seq, precise=precise, **kw)
        e.path = path
        engines.append(e)
        return e
    yield make
    for e in engines:
        e.close()


def feed(e, slot, tok, cuts=None, start=0):
    """Logits of every position of one sequence, fed in portions of the sizes `cuts` (the last repeats)."""
    out, at, i = [], 0, 0
    cuts = cuts or [len(tok)]
    while at < len(tok):
        n = min(cuts[min(i, len(cuts) - 1)], len(tok) - at)
        out.append(e.step_logits(tok[at:at + n], [slot] * n, np.arange(at, at + n) + start, np.arange(n)))
        at, i = at + n, i + 1
    return np.concatenate(out)


def greedy(forward, prompt, total):
    """Greedy ids and the smallest margin between the best two logits on the way."""
    seq, margin = list(prompt), np.inf
    while len(seq) < total:
        lg = forward(np.array(seq))[-1]
        top = np.sort(lg)[-2:]
        margin = min(margin, (top[1] - top[0]) / lg.std())
        seq.append(int(lg.argmax()))
    return seq[len(prompt):], margin


def requests(cfg):
    prompts = [nm.tokens(cfg, n, 80 + n) for n in (5, 1, 23, 9, 40, 2, 17)]
    n_prompt = np.array([len(p) for p in prompts], np.int32)
    ids = np.zeros((len(prompts), n_prompt.max()), np.int32)
    for i, p in enumerate(prompts):
        ids[i, :len(p)] = p
    return prompts, n_prompt, ids
