"""Replay a recorded trace of steps through a model and write logits.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Reads one JSON object per line from standard input:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

All entries of a step run as one batch from the cache that earlier steps left;
requests named in "end" give their pages back after it. If a step wants logits
they are written to OUT/<step>.f32 (little-endian 32-bit floats, in the order of
the entries and of "want"); then the line "done <step>" is printed. Nothing is
sampled.
"""

from __future__ import annotations

import argparse
import json
import os
import sys

MAX_REQUESTS = 4  # sequence slots: requests live at the same time


def main() -> int:
    p = argparse.ArgumentParser(description="Replay a recorded trace of steps through a model and write logits.")
    p.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    p.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    p.add_argument("--out", required=True, help="folder for the logits")
    p.add_argument("--max-tokens", type=int, required=True, help="size of the cache pool in tokens")
    p.add_argument("--device", default="cuda")
    args = p.parse_args()

    if args.device.startswith("cuda"):
        from petals_amd.models.config_base import load_model_config
        from petals_amd.ops.build import build, so_path

        library = load_model_config(args.model).kernel_library
        if not os.path.exists(so_path(library)):
            build(name=library)

    import torch

    from petals_amd.server.local_engine import LocalEngine, Request

    torch.backends.cuda.matmul.allow_tf32 = False
    torch.set_float32_matmul_precision("highest")
    engine = LocalEngine(
        args.model, dtype=getattr(torch, args.dtype), device=torch.device(args.device),
        max_tokens=args.max_tokens, max_requests=MAX_REQUESTS,
    )
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        requests = [Request(e["id"], list(e["tokens"]), list(e.get("want", []))) for e in step["entries"]]
        logits = engine.step(requests) if requests else None
        if logits is not None and logits.shape[0]:
            logits.numpy().astype("<f4").tofile(os.path.join(args.out, f"{step['step']}.f32"))
        for request_id in step.get("end", []):
            engine.end(request_id)
        print(f"done {step['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
