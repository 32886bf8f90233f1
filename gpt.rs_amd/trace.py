"""Replays given token ids through a loaded model, step by step, and hands out logits.

Steps come as JSON objects, one a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

`entries` are the next tokens of each request, run as ONE batch through `model.forward_batch` (the step function that the
generators use) on the caches that earlier steps left; `want` names the places among them whose logits are asked for; `end`
lists the requests whose caches are given back after the step.  Requests of a step either all start or all go on by one
token.
"""
from __future__ import annotations

import json
import os
from typing import Dict, Iterator, List

import numpy as np


class TraceReplay:
    def __init__(self, model):
        self.model = model
        self.live: Dict[str, list] = {}     # request -> its cache slots, one per layer
        self.done: Dict[str, int] = {}      # request -> tokens that have gone through the model

    def step(self, entries: List[dict], end: List[str]) -> np.ndarray:
        """Logits f32 [wanted, vocab] in the order of the entries and of their `want`."""
        ids = [e["id"] for e in entries]
        out = np.zeros((0, self.model.config.vocab_size), np.float32)
        if entries:
            rows, r0 = [], 0
            for e in entries:
                rows += [r0 + int(w) for w in e["want"]]
                r0 += len(e["tokens"])
            for i in ids:
                self.live.setdefault(i, [None] * self.model.num_layers)
            caches = [self.live[i] for i in ids]
            logits = self.model.forward_batch([[int(t) for t in e["tokens"]] for e in entries], [self.done.get(i, 0) for i in ids], caches,
                                              logit_rows=rows or [r0 - 1])
            if rows:
                out = np.asarray(self.model.backend.to_numpy(logits), np.float32)
            else:
                self.model.backend.synchronize()
            for i, e in zip(ids, entries):
                self.done[i] = self.done.get(i, 0) + len(e["tokens"])
        for i in end:
            self.live.pop(i, None)
            self.done.pop(i, None)
        return out


def replay(model, lines: Iterator[str], out_dir: str, emit=print):
    """Runs every step of `lines`; writes <out_dir>/<step>.f32 where something is wanted and emits `done <step>`."""
    run = TraceReplay(model)
    for line in lines:
        if not line.strip():
            continue
        st = json.loads(line)
        got = run.step(st["entries"], st.get("end", []))
        if got.shape[0]:
            got.astype("<f4").tofile(os.path.join(out_dir, f"{st['step']}.f32"))
        emit(f"done {st['step']}")
