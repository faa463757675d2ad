"""Replays a trace of given tokens through a model, step by step, and writes the logits asked for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N < steps

One JSON object per line of standard input: {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [1]}], "end": []}.
A step feeds each entry's tokens to its request -- from what earlier steps left in the cache and the recurrent state -- and
writes the logits at the wanted places to DIR/<step>.f32 ([wanted, vocab], little-endian float32; no file if none are
wanted), then prints "done <step>".  "end" names the requests that give their cache back.  The decoders hold one
sequence, so one request is live at a time.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

import numpy as np


class Replay:
    """The steps of a trace on a model with one sequence."""

    def __init__(self, model):
        self.model, self.live = model, None
        model.reset()

    def step(self, entries, end):
        out = []
        for e in entries:
            if self.live is None:
                self.live = e["id"]
            if e["id"] != self.live:
                raise ValueError(f"request {e['id']!r} starts while {self.live!r} is live (one sequence at a time)")
            if e["tokens"]:
                out.append(self.model.extend(e["tokens"], e.get("want", [])))
        for r in end:
            if r == self.live:
                self.model.reset()
                self.live = None
        return np.concatenate(out) if out else np.empty((0, self.model.cfg.vocab), dtype=np.float32)


def main(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run", description="replay a trace of token ids and write logits")
    ap.add_argument("--model", required=True, help="a folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for the <step>.f32 files")
    ap.add_argument("--max-tokens", type=int, required=True, help="the most tokens that live requests hold at any time")
    a = ap.parse_args(argv)

    from . import build, models, runtime

    build.ensure_library()
    with runtime.Context(0) as ctx:
        model = models.load_model(ctx, a.model, dtype=a.dtype, max_tokens=max(a.max_tokens, 1))
        replay = Replay(model)
        for line in sys.stdin:
            if not line.strip():
                continue
            s = json.loads(line)
            logits = replay.step(s.get("entries", []), s.get("end", []))
            if len(logits):
                logits.astype("<f4").tofile(os.path.join(a.out, f"{s['step']}.f32"))
            print(f"done {s['step']}", flush=True)
        model.free()
    return 0
