"""Replay a trace of given token ids through a model and write logits.

Steps come as JSON lines on standard input:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [1]}],
     "end": []}

Each step is one engine step (LLMEngine.feed): the entries' tokens run as
one batch on the cache and state that earlier steps left.  Wanted logits
go to OUT/<step>.f32 (little-endian f32 [wanted, vocab]); after every
step 'done <step>' is printed.
"""

from __future__ import annotations

import argparse
import json
import os
import sys

# tokens of the KV pool are counted per request in units of this many
POOL_UNIT = 64
MAX_LIVE = 4


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(
        prog="trace_run",
        description="Feed given token ids through a model, step by step, "
                    "and write the logits that each step asks for.")
    ap.add_argument("--model", required=True,
                    help="checkpoint directory (config.json, safetensors)")
    ap.add_argument("--dtype", default="bfloat16",
                    choices=("bfloat16", "float32"))
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="most tokens that live requests hold at a time, "
                         f"each rounded up to {POOL_UNIT}")
    ap.add_argument("--device", default=None,
                    help="torch device (default: the GPU)")
    args = ap.parse_args(argv)

    import torch

    from ..models import (
        build_model, checkpoint_architecture, get_config, get_model_class,
    )
    from .engine import LLMEngine
    from .kv_cache import PagedKVCache

    if checkpoint_architecture(args.model) is None:
        print(f"trace_run: {args.model}/config.json names no known "
              f"architecture", file=sys.stderr)
        return 2
    device = args.device or "cuda:0"
    if device != "cpu":
        if not torch.cuda.is_available():
            print("trace_run: no GPU", file=sys.stderr)
            return 2
    dtype = getattr(torch, args.dtype)
    torch.backends.cuda.matmul.allow_tf32 = False
    torch.set_float32_matmul_precision("highest")
    config = get_config(args.model)
    if device != "cpu":
        from ..ops import build
        build.ensure(get_model_class(args.model).EXTENSIONS)
    pool = -(-args.max_tokens // POOL_UNIT) * POOL_UNIT
    config.fit_positions(max(pool, POOL_UNIT))
    model = build_model(config, weights=args.model, device=device,
                        dtype=dtype)
    block_size = 16
    kv = PagedKVCache.for_model(config, max(1, pool // block_size),
                                device=device, block_size=block_size,
                                kv_dtype=dtype, state_slots=MAX_LIVE)
    engine = LLMEngine(model, kv, max_batch_size=MAX_LIVE)
    os.makedirs(args.out, exist_ok=True)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = engine.feed(
            [(e["id"], e["tokens"], e.get("want", []))
             for e in step["entries"]], step.get("end", []))
        if logits is not None and logits.shape[0]:
            data = logits.cpu().numpy().astype("<f4").tobytes()
            with open(os.path.join(args.out, f"{step['step']}.f32"),
                      "wb") as f:
                f.write(data)
        print(f"done {step['step']}", flush=True)
    return 0
