"""Command line: ``bin/gptoss models | generate | trace``.

  models                     architectures that can be opened
  generate --model PATH ...  greedy generation from token ids through the engine's scheduler
  trace --model DIR ...      replay given tokens step by step and write logits (bin/trace_run)

Nothing here needs PyTorch; what is not compiled yet is compiled first."""
from __future__ import annotations

import argparse
import json
import os
import sys

import numpy as np

from . import build, lib

#: cache slots of a trace: requests that may be live at the same time
TRACE_SLOTS = 8


def architecture_of(path):
    """What config.json of a model folder names; flat files are GPT-OSS."""
    if not os.path.isdir(path):
        return "gpt-oss"
    with open(os.path.join(path, "config.json")) as f:
        return json.load(f).get("architecture")


def open_engine(path, **kw):
    lib.load(path=build.ensure_for(architecture_of(path)))
    from .engine import Engine
    return Engine.open(path, **kw)


def cmd_models(_):
    L = lib.load(path=build.ensure_for("gpt-oss"))
    i = 0
    while (name := L.gptoss_model_name(i)) is not None:
        print(name.decode())
        i += 1
    return 0


def cmd_generate(a):
    prompts = [[int(t) for t in p.split(",")] for p in a.prompt]
    if a.prompts_file:
        with open(a.prompts_file) as f:
            prompts += [[int(t) for t in line.replace(",", " ").split()] for line in f if line.strip()]
    if not prompts:
        sys.exit("generate: give --prompt or --prompts-file")
    longest = max(len(p) for p in prompts)
    total = longest + a.max_new + 1
    eng = open_engine(a.model, max_batch=min(a.batch, len(prompts)), max_seq=total,
                      precise=a.dtype == "float32", keep_logits=False)
    ids = np.zeros((len(prompts), longest), np.int32)
    for i, p in enumerate(prompts):
        ids[i, :len(p)] = p
    n_prompt = np.array([len(p) for p in prompts], np.int32)
    limit = min(total, eng.max_seq + 1)
    out, _ = eng.generate(ids, limit, n_prompt=n_prompt,
                          max_len=None if a.dtype == "float32" and architecture_of(a.model) == "gpt-oss"
                          else np.minimum(n_prompt + a.max_new, limit))
    for row in out:
        end = int(np.argmax(row < 0))
        print(" ".join(str(int(t)) for t in row[:end]))
    return 0


def cmd_trace(a):
    try:
        eng = open_engine(a.model, max_batch=TRACE_SLOTS, max_seq=max(1, a.max_tokens), precise=a.dtype == "float32")
        if eng.info.max_rows == 0:
            raise lib.GptossError(6, "this model has no step over rows in this precision")
    except lib.GptossError as e:
        print(f"trace: {e}", file=sys.stderr)
        return 3 if a.dtype == "float32" and e.code == 6 else 1
    live = {}    # request id -> [cache slot, positions so far]
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        tokens, slots, positions, want = [], [], [], []
        for entry in step["entries"]:
            if entry["id"] not in live:
                live[entry["id"]] = [eng.acquire_slot(), 0]
            slot, at = live[entry["id"]]
            n = len(entry["tokens"])
            want += [len(tokens) + w for w in entry.get("want", ())]
            tokens += entry["tokens"]
            slots += [slot] * n
            positions += range(at, at + n)
            live[entry["id"]][1] = at + n
        # rows are wanted in ascending order; the file has them in the order they were asked for
        order = sorted(set(want))
        if tokens:
            logits = eng.step_logits(tokens, slots, positions, order)
            if want:
                at = {w: i for i, w in enumerate(order)}
                logits[[at[w] for w in want]].astype("<f4").tofile(os.path.join(a.out, f"{step['step']}.f32"))
        for r in step.get("end", ()):
            if r in live:
                eng.release_slot(live.pop(r)[0])
        print(f"done {step['step']}", flush=True)
    eng.close()
    return 0


def main(argv=None):
    ap = argparse.ArgumentParser(prog="gptoss", description=__doc__.split("\n")[0])
    sub = ap.add_subparsers(dest="cmd", required=True)
    sub.add_parser("models", help="architectures that can be opened").set_defaults(run=cmd_models)
    g = sub.add_parser("generate", help="greedy generation from token ids")
    g.add_argument("--model", required=True, help="folder with config.json and model.safetensors, or a .bin file")
    g.add_argument("--prompt", action="append", default=[], help="token ids with commas between them (repeatable)")
    g.add_argument("--prompts-file", help="one prompt of token ids a line")
    g.add_argument("--max-new", type=int, default=32)
    g.add_argument("--batch", type=int, default=64, help="sequences decoded together")
    g.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    g.set_defaults(run=cmd_generate)
    t = sub.add_parser("trace", help="replay tokens step by step from standard input, write logits")
    t.add_argument("--model", required=True)
    t.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    t.add_argument("--out", required=True, help="folder for <step>.f32")
    t.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold")
    t.set_defaults(run=cmd_trace)
    a = ap.parse_args(argv)
    return a.run(a)
