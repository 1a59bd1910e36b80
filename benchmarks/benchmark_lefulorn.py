"""Prefill and decode throughput of Lefulorn layers beside BLOOM layers of equal
size (the closest family: distance bias, biased projections, a two-matrix MLP),
random weights, one GPU.

Run through `bench.py --compare lefulorn`. Each side runs a stack of equal layers
with the step function that serves it: Lefulorn through the span engine (decode:
its captured graph), BLOOM through its fused blocks (decode: the per-session span
graph). `attention` and `delta` are the two mixers, each with a feed-forward.
Prints one JSON line per size and batch.
"""

from __future__ import annotations

import json

import torch

from benchmarks.benchmark_tulezen import build, timed

SIZES = {
    "2k": dict(width=2048, heads=16, dim=128, ff=8192, window=1024),
    "4k": dict(width=4096, heads=32, dim=128, ff=16384, window=1024),
    "8k": dict(width=8192, heads=64, dim=128, ff=32768, window=1024),
}
LAYERS, PREFILL, CONTEXT = 4, 2048, 2048
FAMILIES = ("attention", "delta", "bloom")


def lefulorn_config(s, kind):
    from petals_amd.models.lefulorn.config import LefulornConfig

    sizes = {"heads": s["heads"], "kv_heads": s["heads"], "dim": s["dim"], "vdim": s["dim"]}
    if kind == "delta":
        layer = {"type": "channel_delta", "mixer": {**sizes, "conv": 4}}
    else:
        layer = {"type": "attention", "mixer": {
            **sizes, "scale": s["dim"] ** -0.5, "mask": {"size": s["window"]}, "q_temp": {"coef": 0.1, "every": 512},
            "v_mix": True,
        }}
    layer["mlp"] = {"kind": "dense", "ff": s["ff"]}
    return LefulornConfig.from_hf_dict(
        {"layers": [layer] * LAYERS, "norm": {"eps": 1e-6}, "vocab": 1024, "width": s["width"]}, name_or_path="bench"
    )


def bloom_config(s):
    from petals_amd.models.bloom.config import BloomConfig

    return BloomConfig(
        hidden_size=s["width"], num_hidden_layers=LAYERS, num_attention_heads=s["heads"], intermediate_size=s["ff"],
        vocab_size=1024, max_position_embeddings=8192, name_or_path="bench",
    )


def engine_runs(config, device, batch):
    """(prefill callable, decode callable) of a paged family's layers"""
    from petals_amd.server.span_engine import SpanEngine, StepEntry

    blocks = build(config, device)
    length = CONTEXT + 64 * 8
    pool = SpanEngine.pool_for(blocks, (batch + 1) * length, dtype=torch.bfloat16, device=device, max_sequences=batch + 1)
    engine = SpanEngine(dict(enumerate(blocks)), pool, max_length=length)
    uids = tuple(range(LAYERS))
    x = torch.randn(PREFILL, config.stream_width, device=device)
    sequences = [pool.open() for _ in range(batch)]
    other = pool.open()
    for q in sequences:
        engine.step(uids, [StepEntry(q, x, 0)])

    def prefill():
        engine.step(uids, [StepEntry(other, x, 0)])

    def decode():
        engine.step(uids, [StepEntry(q, x[:1], q.length) for q in sequences])

    return prefill, decode


def bloom_runs(s, device, batch):
    from petals_amd.server.handler import _SpanDecodeGraph

    blocks = build(bloom_config(s), device)
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
def main(steps: int = 20, warmup: int = 5, sizes=None, families=FAMILIES, batches=(1, 8)):
    device = torch.device("cuda", 0)
    for name in sizes or SIZES:
        s = SIZES[name]
        for batch in batches:
            row = {"size": name, "layers": LAYERS, "batch": batch, "prefill_tokens": PREFILL, "context": CONTEXT}
            for f in families:  # in turn, on the same box
                runs = bloom_runs(s, device, batch) if f == "bloom" else engine_runs(lefulorn_config(s, f), device, batch)
                prefill, decode = runs
                if batch == 1:
                    row[f"{f}_prefill_tok_s"] = round(PREFILL / timed(prefill, max(3, steps // 4), 2))
                t = timed(decode, steps, warmup)
                row[f"{f}_decode_tok_s"] = round(batch / t)
                row[f"{f}_decode_us_per_layer"] = round(1e6 * t / LAYERS, 1)
                del runs, prefill, decode
                torch.cuda.empty_cache()
            print(json.dumps(row), flush=True)


if __name__ == "__main__":
    import sys

    main(
        sizes=[a for a in sys.argv[1:] if a in SIZES] or None,
        families=tuple(a for a in sys.argv[1:] if a in FAMILIES) or FAMILIES,
        batches=tuple(int(a) for a in sys.argv[1:] if a.isdigit()) or (1, 8),
    )
