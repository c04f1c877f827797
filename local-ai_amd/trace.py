"""Replays a trace: token ids come in as steps, one JSON object a line on standard input, and the logits that a step asks for
go to files.  Nothing is sampled.

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": ["a"]}

Each entry continues its request's sequence; `end` gives requests' slots back after the step.  A step with wanted places
writes DIR/<step>.f32, little-endian f32 [wanted, vocab] in the order of the entries; every step prints ``done <step>``."""
from __future__ import annotations

import argparse
import json
import os
import sys
from typing import Dict

import numpy as np

from . import BF16, F32
from .registry import load_model

DTYPES = {"bfloat16": BF16, "float32": F32}


def replay(model, lines, out_dir: str, emit) -> None:
    live: Dict[str, object] = {}
    for line in lines:
        line = line.strip()
        if not line:
            continue
        step = json.loads(line)
        parts = []
        for e in step["entries"]:
            if e["id"] not in live:
                live[e["id"]] = model.new_sequence()
            got = model.step(live[e["id"]], e["tokens"], e.get("want", []))
            if len(got):
                parts.append(got)
        if parts:
            path = os.path.join(out_dir, f"{step['step']}.f32")
            np.concatenate(parts).astype("<f4").tofile(path)
        for i in step.get("end", []):
            if i in live:
                model.end_sequence(live.pop(i))
        emit(f"done {step['step']}")


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=sorted(DTYPES), default="bfloat16", help="activations and caches")
    ap.add_argument("--out", required=True, help="folder the logits are written to")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold at any time")
    ap.add_argument("--sequences", type=int, default=64, help="most requests live at any time")
    a = ap.parse_args(argv)
    model = load_model(a.model, a.max_tokens, DTYPES[a.dtype], max_sequences=a.sequences)

    def emit(text):
        print(text, flush=True)
    replay(model, sys.stdin, a.out, emit)
    return 0
