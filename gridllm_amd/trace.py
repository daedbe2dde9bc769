"""Replay a trace of token ids through a model and write the logits asked for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

DIR holds config.json and model.safetensors of a model with mixed steps. Steps
come on standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [1]}],
     "end": []}

`entries` are the requests' next tokens, run as one batch; `want` the places
among them whose logits are written, f32 [wanted, vocab], to <out>/<step>.f32;
`end` the requests that are done after the step. Every step is acknowledged by
the line "done <step>". A request is admitted at its first entry and keeps its
slot until it ends; at most SLOTS are live at once, and their tokens, each
request's rounded up to pages of 64, may add up to --max-tokens.

The engine does all of it: its loader, cache and slots, and the step function
that generation runs on (decode-only steps go through the captured graphs).
"""

from __future__ import annotations

import argparse
import json
import os
import sys
from typing import IO, Optional

SLOTS = 4
_DTYPES = {"bfloat16": "bf16", "float32": "fp32"}


def make_engine(model: str, dtype: str, max_tokens: int, device: str):
    import torch

    from gridllm_amd.config import EngineConfig
    from gridllm_amd.engine import InferenceEngine
    torch.backends.cuda.matmul.allow_tf32 = False
    torch.set_float32_matmul_precision("highest")
    engine = InferenceEngine(EngineConfig(
        weights_path=model, dtype=_DTYPES[dtype], device=device,
        max_seq_len=0, max_batch_size=SLOTS, kv_tokens=max_tokens,
        autotune=False, context_shift=False))
    if not engine.mixed:
        raise SystemExit(f"{model}: {engine.spec.name} has no mixed steps")
    return engine


def replay(engine, steps: IO[str], out: str, acks: IO[str]) -> None:
    """Run the steps of `steps` line by line."""
    slots: dict[str, int] = {}
    for line in steps:
        if not line.strip():
            continue
        step = json.loads(line)
        entries = []
        for e in step["entries"]:
            if e["id"] not in slots:
                slots[e["id"]] = engine.open_sequence()
            entries.append((slots[e["id"]], e["tokens"], e["want"]))
        if entries:
            logits = engine.run_step(entries)
            if logits.shape[0]:
                logits.cpu().numpy().astype("<f4").tofile(
                    os.path.join(out, f"{step['step']}.f32"))
        for rid in step["end"]:
            if rid in slots:
                engine.close_sequence(slots.pop(rid))
        print(f"done {step['step']}", file=acks, flush=True)


def main(argv: Optional[list[str]] = None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=(
        "Replay token ids step by step and write logits."))
    ap.add_argument("--model", required=True,
                    help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=sorted(_DTYPES), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="size of the KV pool, in tokens")
    ap.add_argument("--device", default="cuda:0",
                    help="cuda:N, or cpu for the PyTorch reference in f32")
    args = ap.parse_args(argv)
    os.environ.setdefault("LOG_LEVEL", "warn")
    if args.device != "cpu":
        from gridllm_amd.models.registry import spec_from_dir
        from gridllm_amd.ops.build import build, libs_of
        spec = spec_from_dir(args.model)
        # compiles what the model needs and is missing or stale
        build(names=libs_of(spec) if spec else None)
    engine = make_engine(args.model, args.dtype, args.max_tokens, args.device)
    replay(engine, sys.stdin, args.out, sys.stdout)
    return 0


if __name__ == "__main__":
    raise SystemExit(main())
