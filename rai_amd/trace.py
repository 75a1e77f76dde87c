"""Replays a trace of token ids through a model and writes logits (the program behind bin/trace_run).

One JSON object a line on standard input:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

Each step appends its entry's tokens to that request's context; `want` names the tokens of the entry whose logits go to
OUT/<step>.f32 (little-endian f32, [wanted, vocab]).  "done <step>" follows on standard output.  Nothing is sampled.  A
request holds the decoder's cache from its first token until a step lists it under `end`; requests follow one another.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

import numpy as np


def run(args, lines, out):
    from .config import load_model

    dec = load_model(args.model, {"bfloat16": "bf16", "float32": "f32"}[args.dtype], max_context=args.max_tokens)
    live = None   # the request whose context the cache holds
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        wanted = []
        for e in step["entries"]:
            if live not in (None, e["id"]):
                raise ValueError(f"step {step['step']}: request {e['id']!r} starts while {live!r} is live")
            live = e["id"]
            wanted.append(dec.forward_rows(np.array([e["tokens"]], np.uint32), e["want"]))
        rows = sum(w.shape[0] for w in wanted)
        if rows:
            path = os.path.join(args.out, f"{step['step']}.f32")
            np.concatenate(wanted).astype("<f4").tofile(path)
        if live in step["end"]:
            dec.clear_kv_cache()
            live = None
        print(f"done {step['step']}", file=out, flush=True)
    dec.close()


def main(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run", description="Replay a trace of token ids through a model and write logits.")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, default=None, help="most tokens that live requests hold at any time")
    run(ap.parse_args(argv), sys.stdin, sys.stdout)
    return 0


if __name__ == "__main__":
    sys.exit(main())
