"""Replay a trace of given tokens through the engine and write the logits it asks for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N < steps.jsonl

Steps come on standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

`entries` are the next tokens of each request (one batch), `want` the places among them whose logits are written to
OUT/<step>.f32 (little-endian f32, [wanted, vocab], in the order of the entries); `end` lists requests that are finished
after the step. Each step is answered with a line `done <step>`. The tokens go through Engine.feed: the engine's own block
pool (N tokens), state slots (four live requests), step functions and kernels."""
from __future__ import annotations

import argparse
import json
import os
import sys

BLOCK = 16
MAX_LIVE = 4
CHUNK = 2048          # rows per forward; longer steps run in several
LOGIT_ROWS = 256


def parse(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run", description="replay a token trace and write logits")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder of the logit files")
    ap.add_argument("--max-tokens", type=int, required=True, help="tokens that live requests hold at most")
    ap.add_argument("--device", default="cuda:0")
    return ap.parse_args(argv)


def build_engine(args):
    import torch

    from . import build
    from .engine.engine import Engine
    from .models.registry import checkpoint_kind, load_model
    if checkpoint_kind(args.model) != "stack":
        raise SystemExit("trace_run: --model needs a folder with config.json and model.safetensors")
    if not build.stack_current():
        build.build_stack()
    blocks = -(-args.max_tokens // BLOCK)
    model = load_model(args.model, args.device, dtype=getattr(torch, args.dtype), ctx=blocks * BLOCK)
    chunk = max(64, min(CHUNK, blocks * BLOCK))
    return Engine(model, None, max_batch=MAX_LIVE, block_size=BLOCK, num_blocks=blocks, max_prefill_tokens=chunk,
                  max_logit_rows=min(LOGIT_ROWS, chunk))


def replay(eng, lines, out_dir: str, reply):
    import torch
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        entries = [(e["id"], e["tokens"], e.get("want", [])) for e in step["entries"]]
        got = eng.feed(entries) if entries else []
        rows = torch.cat(got) if got else torch.zeros(0, 0)
        if rows.shape[0]:
            rows.numpy().astype("<f4").tofile(os.path.join(out_dir, f"{step['step']}.f32"))
        for rid in step.get("end", []):
            eng.feed_end(rid)
        reply(f"done {step['step']}")


def main(argv=None) -> int:
    args = parse(argv)
    eng = build_engine(args)
    # what the steps print (compiler output of a first call included) must not look like an answer
    replay(eng, sys.stdin, args.out, lambda s: print(s, flush=True))
    return 0


if __name__ == "__main__":
    sys.exit(main())
