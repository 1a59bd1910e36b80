"""Prefill and decode throughput of Tulezen layers beside Mixtral layers of equal
size (the closest family: attention + routed experts), random weights, one GPU.

Run through `bench.py --compare tulezen`. Each side runs a stack of equal layers
with the step function that serves it: Tulezen through the span engine (decode:
its captured graph), Mixtral through its fused blocks (decode: the per-session
span graph). Prints one JSON line per size.
"""

from __future__ import annotations

import json
import time

import torch

# width, heads, head size, kv heads (mixtral) / latent (tulezen), window, experts, top, ff
SIZES = {
    "2k-8x4k": dict(width=2048, heads=16, dim=128, kv_heads=4, rank=512, window=1024, experts=8, top=2, ff=4096),
    "4k-8x14k": dict(width=4096, heads=32, dim=128, kv_heads=8, rank=512, window=1024, experts=8, top=2, ff=14336),
    "2k-64x1k": dict(width=2048, heads=16, dim=128, kv_heads=4, rank=256, window=512, experts=64, top=4, ff=1408),
}
LAYERS, PREFILL, CONTEXT = 4, 2048, 2048


def tulezen_config(s):
    from petals_amd.models.tulezen.config import TulezenConfig

    layer = {
        "type": "latent_attention",
        "mixer": {"heads": s["heads"], "dim": s["dim"], "vdim": s["dim"], "kv_rank": s["rank"],
                  "scale": s["dim"] ** -0.5, "mask": {"size": s["window"]}},
        "mlp": {"kind": "moe", "expert": {"ff": s["ff"], "limit": 7.0},
                "router": {"experts": s["experts"], "top": s["top"]}},
    }
    return TulezenConfig.from_hf_dict(
        {"layers": [layer] * LAYERS, "norm": {"eps": 1e-6}, "vocab": 1024, "width": s["width"]}, name_or_path="bench"
    )


def mixtral_config(s):
    from petals_amd.models.mixtral.config import MixtralConfig

    return MixtralConfig(
        hidden_size=s["width"], num_hidden_layers=LAYERS, num_attention_heads=s["heads"],
        num_key_value_heads=s["kv_heads"], intermediate_size=s["ff"], vocab_size=1024,
        max_position_embeddings=8192, num_local_experts=s["experts"], num_experts_per_tok=s["top"],
        head_dim_override=s["dim"], name_or_path="bench",
    )


def build(config, device):
    from petals_amd.server.from_pretrained import build_empty_block, init_random_block_

    blocks = []
    for i in range(LAYERS):
        block = build_empty_block(config, i, device, torch.bfloat16)
        init_random_block_(block, config, i)
        blocks.append(block.eval().optimize_for_inference())
    return blocks


def timed(fn, steps, warmup):
    for _ in range(warmup):
        fn()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(steps):
        fn()
    torch.cuda.synchronize()
    return (time.perf_counter() - t0) / steps


def tulezen_runs(s, device, batch):
    """(prefill callable, decode callable)"""
    from petals_amd.server.span_engine import SpanEngine, StepEntry

    blocks = build(tulezen_config(s), device)
    length = CONTEXT + 64
    pool = SpanEngine.pool_for(blocks, batch * length, dtype=torch.bfloat16, device=device)
    engine = SpanEngine(dict(enumerate(blocks)), pool, max_length=length)
    uids = tuple(range(LAYERS))
    x = torch.randn(PREFILL, s["width"], device=device)
    sequences = [pool.open() for _ in range(batch)]
    for q in sequences:
        engine.step(uids, [StepEntry(q, x, 0)])

    def prefill():
        engine.step(uids, [StepEntry(sequences[0], x, 0)])

    def decode():
        engine.step(uids, [StepEntry(q, x[:1], CONTEXT) for q in sequences])

    return prefill, decode


def mixtral_runs(s, device, batch):
    from petals_amd.server.handler import _SpanDecodeGraph

    blocks = build(mixtral_config(s), device)
    shape, _ = blocks[0].kv_cache_shape(batch, CONTEXT + 64)
    caches = [tuple(torch.zeros(shape, device=device, dtype=torch.bfloat16) for _ in range(2)) for _ in blocks]
    x = torch.randn(batch, PREFILL, s["width"], device=device, dtype=torch.bfloat16)
    one = [(k[:1].contiguous(), v[:1].contiguous()) for k, v in caches]

    def forward(h, kv):
        for block, c in zip(blocks, kv):
            h = block(h, kv_cache=c, prefix_length=0)

    forward(x, caches)
    graph = _SpanDecodeGraph(blocks, caches, batch, s["width"], device, torch.bfloat16, None, CONTEXT)

    def prefill():
        forward(x[:1], one)

    def decode():
        graph.step(x[:, :1], CONTEXT)

    return prefill, decode


@torch.inference_mode()
def main(steps: int = 20, warmup: int = 5, sizes=None, families=("tulezen", "mixtral")):
    device = torch.device("cuda", 0)
    runs = {"tulezen": tulezen_runs, "mixtral": mixtral_runs}
    for name in sizes or SIZES:
        s = SIZES[name]
        for batch in (1, 8):
            if batch * s["top"] > 16:
                batch = 16 // s["top"]  # the mixtral decode path's routed rows
            row = {"size": name, "layers": LAYERS, "batch": batch, "prefill_tokens": PREFILL, "context": CONTEXT}
            made = {f: runs[f](s, device, batch) for f in families}
            for f in families:  # in turn, on the same box
                prefill, decode = made[f]
                if batch == 1:
                    row[f"{f}_prefill_tok_s"] = round(PREFILL / timed(prefill, max(3, steps // 4), 2))
                t = timed(decode, steps, warmup)
                row[f"{f}_decode_tok_s"] = round(batch / t)
                row[f"{f}_decode_us_per_layer"] = round(1e6 * t / LAYERS, 1)
            print(json.dumps(row), flush=True)
            del made
            torch.cuda.empty_cache()


if __name__ == "__main__":
    import os
    import sys

    sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
    names = [a for a in sys.argv[1:] if a in SIZES] or None
    fams = tuple(a for a in sys.argv[1:] if a in ("tulezen", "mixtral")) or ("tulezen", "mixtral")
    main(sizes=names, families=fams)
