"""Replays a trace of token portions through a decoder and writes the logits asked for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Steps come on standard input, one JSON object a line: {"step", "entries": [{"id", "tokens", "want"}], "end": [ids]}.
DIR/<step>.f32 receives the wanted logits as little-endian f32 rows; `done <step>` follows on standard output.  The
decoder holds one sequence at a time, so a request ends before the next one starts.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

import numpy as np


class Sequences:
    """Which request occupies the decoder's cache, and up to where."""

    def __init__(self, model):
        self.model, self.id, self.length = model, None, 0

    def feed(self, rid: str, tokens, want) -> np.ndarray:
        if self.id is None:
            self.id, self.length = rid, 0
        elif self.id != rid:
            raise ValueError(f"request {rid} starts while {self.id} is live: the cache holds one sequence")
        if not tokens:
            raise ValueError(f"request {rid}: a step without tokens")
        if self.length + len(tokens) > self.model.max_pos:
            raise ValueError(f"request {rid} has more than {self.model.max_pos} tokens")
        logits = self.model.feed(tokens, self.length, want)
        self.length += len(tokens)
        return logits

    def end(self, rid: str):
        if rid == self.id:
            self.id, self.length = None, 0


def replay(model, lines, out_dir: str, done) -> None:
    sequences = Sequences(model)
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        rows = [sequences.feed(e["id"], e["tokens"], e.get("want") or []) for e in step.get("entries", [])]
        if any(len(r) for r in rows):
            path = os.path.join(out_dir, f"{step['step']}.f32")
            np.concatenate([r for r in rows if len(r)]).astype("<f4").tofile(path)
        for rid in step.get("end", []):
            sequences.end(rid)
        done(step["step"])


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="Replay a trace of token portions and write logits.")
    ap.add_argument("--model", required=True, help="model folder, or a GGUF file")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16", help="number format of the activations")
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, default=4096, help="positions the cache has room for")
    args = ap.parse_args(argv)

    from . import hip, models
    dev = hip.Device(0)
    try:
        model = models.load(dev, args.model, max_pos=max(args.max_tokens, 1),
                            act=hip.ACT_F32 if args.dtype == "float32" else hip.ACT_BF16)
    except models.UnsupportedFormat as e:
        print(f"trace_run: {e}", file=sys.stderr)
        return 3
    os.makedirs(args.out, exist_ok=True)
    replay(model, sys.stdin, args.out, lambda n: print(f"done {n}", flush=True))
    model.free()
    dev.close()
    return 0
