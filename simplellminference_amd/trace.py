"""Trace replay: given token ids run through a model step by step, and the logits at wanted places are written out
(``bin/trace_run``). A step is one batch of requests: all at their first token, or all one token further; it runs
through the model's own ``feed`` on the caches and states the earlier steps left.

Input: one JSON object a line, ``{"step": n, "entries": [{"id", "tokens", "want"}], "end": [ids]}``. Output: for a step
with wanted places ``<out>/<step>.f32`` (little-endian fp32 [wanted, vocab], in entry order), and a line ``done <step>``
after every step."""
from __future__ import annotations

import argparse
import json
import os
import sys

import numpy as np

from .registry import load_model
from .sequences import SlotMap


class TraceRunner:
    def __init__(self, folder: str, dtype: str, max_tokens: int, batch: int = 1):
        self.folder, self.dtype, self.max_tokens = folder, dtype, max_tokens
        self.model, self.slots = None, SlotMap(0)
        self._open(batch)

    def _open(self, batch: int):
        """A model with room for `batch` sequences (a larger batch than before, between batches: loaded anew)."""
        if self.model is not None:
            self.model.close()
        self.model = load_model(self.folder, self.dtype, self.max_tokens, batch)
        self.slots = SlotMap(batch)

    def step(self, entries: list[dict], end: list[str]) -> np.ndarray:
        new = [e for e in entries if e["id"] not in self.slots]
        if len(self.slots) + len(new) > self.slots.capacity:
            if len(self.slots):
                raise RuntimeError("a request joins a full batch")
            self._open(len(new))
        for e in new:
            self.slots.begin(e["id"])
        at = [self.slots.advance(e["id"], len(e["tokens"])) for e in entries]
        out = np.empty((0, self.model.local_vocab), np.float32)
        if entries:
            wants = [sorted(set(e["want"])) for e in entries]
            out = self.model.feed([a[0] for a in at], [a[1] for a in at], [e["tokens"] for e in entries], wants)
            order, base = [], 0
            for e, w in zip(entries, wants):  # rows back in the order asked for
                order += [base + w.index(p) for p in e["want"]]
                base += len(w)
            out = out[order]
        for rid in end:
            self.slots.end(rid)
        return out


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.splitlines()[0])
    ap.add_argument("--model", required=True, help="folder with config.json and the weights")
    ap.add_argument("--dtype", required=True, choices=("bfloat16", "float32"))
    ap.add_argument("--out", required=True, help="folder for the logits files")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold together")
    a = ap.parse_args(argv)
    run = TraceRunner(a.model, a.dtype, a.max_tokens)
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        got = run.step(s["entries"], s.get("end", []))
        if len(got):
            got.astype("<f4").tofile(os.path.join(a.out, f"{s['step']}.f32"))
        print(f"done {s['step']}", flush=True)
    return 0
