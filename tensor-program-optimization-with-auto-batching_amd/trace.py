"""Replays a trace of token ids through a model, step by step, and writes the logits that the trace asks for.

    trace_run --model DIR --dtype bfloat16|float32|float16 --out DIR --max-tokens N

Steps come on standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

`entries`: for each request its next tokens and the places among them whose logits are wanted; `end`: the requests that are
finished after the step, whose pages and slots are given back.  Wanted logits go to DIR/<step>.f32 in the order of the
entries and of `want` ([wanted, vocab], little-endian fp32); after every step the line `done <step>` is printed.  Nothing
is sampled.  Exit code 3: the model does not run in the element type asked for.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

import numpy as np
import torch

from . import build, registry
from .kv_cache import PAGE


class TraceRunner:
    def __init__(self, model, max_tokens: int, max_requests: int = 64):
        self.model = model
        self.kv = model.create_paged_kv_cache(max_requests, max_tokens, max_tokens, PAGE, max_seq_len=max_tokens + PAGE)

    def step(self, entries, end=()):
        """-> wanted logits [n, vocab] (host), or None when nothing is wanted."""
        kv, out = self.kv, None
        entries = [e for e in entries if e["tokens"]]
        if entries:
            for e in entries:
                if e["id"] not in kv.slot:
                    kv.add_sequence(e["id"])
            lens = [len(e["tokens"]) for e in entries]
            starts = np.concatenate([[0], np.cumsum(lens)[:-1]])
            rows = [int(s) + int(w) for s, e in zip(starts, entries) for w in e.get("want", ())]
            ids = torch.tensor([t for e in entries for t in e["tokens"]], dtype=torch.int32)
            kv.begin_forward([e["id"] for e in entries], lens)
            hidden = self.model["embed"](ids)
            logits = self.model.forward(hidden, kv, None, torch.tensor(rows, dtype=torch.int64, device=self.model.device))
            kv.end_forward()
            if rows:
                out = logits.cpu().numpy()
        for sid in end:
            if sid in kv.slot:
                kv.free_sequence(sid)
        return out


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.split("\n")[0])
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", required=True, choices=["bfloat16", "float32", "float16"])
    ap.add_argument("--out", required=True, help="folder the logits are written to")
    ap.add_argument("--max-tokens", required=True, type=int, help="most tokens that live requests hold at any time")
    a = ap.parse_args(argv)
    cls = registry.model_class(registry.read_config(a.model))
    if a.dtype not in cls.dtypes:
        print(f"{cls.__name__} runs in {', '.join(cls.dtypes)}, not in {a.dtype}", file=sys.stderr)
        return 3
    build.ensure(a.dtype)
    runner = TraceRunner(registry.load_model(a.model, a.dtype), a.max_tokens)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = runner.step(step["entries"], step.get("end", ()))
        if logits is not None:
            np.ascontiguousarray(logits, dtype="<f4").tofile(os.path.join(a.out, f"{step['step']}.f32"))
        print(f"done {step['step']}", flush=True)
    return 0
