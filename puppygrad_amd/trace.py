"""Replays a trace of requests on a model: each step brings the next tokens of a request, and the
logits of the places it asks for are written out.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N < steps

A step is one line of JSON on standard input,

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": ["a"]}

with `want` the places among `tokens` whose logits are wanted.  They go to OUT/<step>.f32 as
little-endian f32, [wanted][vocab], in the order of the entries and of `want`; the line
`done <step>` follows on standard output.  Requests in `end` give their cache back.

Every portion runs through Model.extend, the same step, caches and kernels a generation uses.
bfloat16 keeps the weights in bf16 (activations and state are f32), float32 keeps them in f32 and
all products are exact f32 products.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
from typing import Dict, List

import numpy as np

from . import _lib
from .model import Gpt2HipConfig, KvCache
from .models import load_model

STORAGE = {"bfloat16": _lib.PG_STORE_BF16, "float32": _lib.PG_STORE_F32}


class TraceRunner:
    """The live requests of a trace, a cache each; freed caches are used again."""

    def __init__(self, model):
        self.model = model
        self.live: Dict[str, KvCache] = {}
        self.free: List[KvCache] = []

    def _cache(self, request: str) -> KvCache:
        if request not in self.live:
            cache = self.free.pop() if self.free else self.model.new_kv_cache()
            cache.clear()
            self.live[request] = cache
        return self.live[request]

    def step(self, step: dict) -> np.ndarray:
        """Runs one step; the wanted logits, [wanted][vocab]."""
        rows = [np.empty((0, self.model.vocab_size), np.float32)]
        for entry in step["entries"]:
            want = [int(w) for w in entry["want"]]
            places = sorted(set(want))
            if not entry["tokens"]:
                continue
            logits = self.model.extend(entry["tokens"], self._cache(entry["id"]), places)
            if want:
                got = logits.to_host().reshape(len(places), -1)
                rows.append(got[[places.index(w) for w in want]])
        for request in step.get("end", []):
            if request in self.live:
                self.free.append(self.live.pop(request))
        return np.concatenate(rows)


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(description=__doc__.split("\n\n")[0])
    ap.add_argument("--model", required=True, help="directory with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=sorted(STORAGE), default="bfloat16")
    ap.add_argument("--out", required=True, help="directory for the logits")
    ap.add_argument("--max-tokens", type=int, default=0,
                    help="most tokens that live requests hold at a time (caches size themselves)")
    args = ap.parse_args(argv)
    runner = TraceRunner(load_model(args.model, Gpt2HipConfig(weight_storage=STORAGE[args.dtype])))
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        rows = runner.step(step)
        if len(rows):
            rows.astype("<f4").tofile(os.path.join(args.out, f"{step['step']}.f32"))
        print(f"done {step['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
