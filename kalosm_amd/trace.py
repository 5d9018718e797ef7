"""Replays recorded token ids through a decoder: steps come in as JSON lines, the logits of the places a step names leave as
little-endian f32 files.  Sequences are replayed one after the other, each continuing on the decoder's caches."""
from __future__ import annotations

import json
import os
import sys

import numpy as np

from . import registry
from .fusor import Device


class TraceError(ValueError):
    pass


class Replay:
    def __init__(self, model, out_dir: str):
        self.model, self.out_dir, self.live = model, out_dir, None

    def step(self, step: dict) -> None:
        rows = []
        for entry in step["entries"]:
            name, want = entry["id"], entry["want"]
            if self.live is not None and self.live != name:
                raise TraceError(f"request {name!r} starts before {self.live!r} has ended: one sequence at a time")
            if self.live is None:
                self.model.reset()
                self.live = name
            logits = self.model.forward(entry["tokens"], want=want)
            if len(want):
                rows.append(logits)
        if rows:
            path = os.path.join(self.out_dir, f"{step['step']}.f32")
            np.concatenate(rows).astype("<f4").tofile(path)
        for name in step.get("end", []):
            if name == self.live:
                self.model.reset()
                self.live = None


def run(model_path: str, dtype: str, out_dir: str, max_tokens: int, lines=None, out=None) -> int:
    lines, out = lines or sys.stdin, out or sys.stdout
    device = Device.gpu(0)
    # a context below 40 positions could not be trimmed to its tail
    replay = Replay(registry.load(device, model_path, dtype=dtype, ctx=max(int(max_tokens), 64)), out_dir)
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        replay.step(step)
        print(f"done {step['step']}", file=out, flush=True)
    return 0
