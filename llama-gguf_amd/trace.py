"""Replays a trace: steps of given token ids through a model, logits written where they are asked for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR [--max-tokens N]

A step is one JSON line on standard input, ``{"step": 0, "entries": [{"id": "a", "tokens": [..], "want": [..]}], "end": ["a"]}``: the
next tokens of a request, the places among them whose logits are wanted, and the requests that are over.  Logits go to
``DIR/<step>.f32`` (little-endian, [wanted, vocab]); ``done <step>`` is printed after every step.  Requests come one after the other:
the context is reset when a new one begins.  Everything runs through ``HipGpuInference.eval`` — prompt portions as blocks, single
tokens as the replayed token graph that greedy decoding uses.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

import numpy as np

from . import hip_backend as hb
from .layered_model import load_model


class TraceRunner:
    def __init__(self, gpu: hb.HipGpuInference):
        self.gpu, self.active = gpu, None

    def step(self, entries, end) -> np.ndarray:
        rows = []
        for e in entries:
            if e["id"] != self.active:
                if self.active is not None:
                    raise hb.BackendError(5, f"request {e['id']!r} starts while {self.active!r} is still live: one sequence per context")
                self.gpu.reset()
                self.active = e["id"]
            if e["tokens"]:
                rows.append(self.gpu.eval(e["tokens"], e["want"]))
        if self.active in end:
            self.active = None
        return np.concatenate(rows) if rows else np.empty((0, self.gpu.vocab_size), np.float32)


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="replay token portions through a model and write logits")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, default=8192, help="most tokens a live request holds")
    ap.add_argument("--device", type=int, default=0)
    a = ap.parse_args(argv)
    gpu = load_model(a.model, max(a.max_tokens, 1), a.device, hb.COMPUTE_F32 if a.dtype == "float32" else hb.COMPUTE_BF16)
    run = TraceRunner(gpu)
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = run.step(s["entries"], s.get("end", []))
        if logits.shape[0]:
            logits.astype("<f4").tofile(os.path.join(a.out, f"{s['step']}.f32"))
        print(f"done {s['step']}", flush=True)
    gpu.close()
    return 0
