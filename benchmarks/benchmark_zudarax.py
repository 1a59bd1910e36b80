"""Prefill and decode throughput of Zudarax layers beside layers of equal size of the
closest families, random weights, one GPU.

Run through `bench.py --compare zudarax`. Each side runs a stack of equal layers with
the span engine that serves it (decode: its captured graph), with a feed-forward of
4x width:

  capped, paired, sigmoid   the three kinds of attention; paired with half the heads and
                            values of twice the size, as it has two maps per head. Chunks
                            are longer than the context, so that all see the same keys
  attention, delta          Lefulorn's two mixers (attention over all earlier tokens here)

Prints one JSON line per size and batch.
"""

from __future__ import annotations

import json

import torch

from benchmarks.benchmark_lefulorn import CONTEXT, LAYERS, PREFILL, engine_runs, lefulorn_config
from benchmarks.benchmark_tulezen import timed

SIZES = {
    "2k": dict(width=2048, heads=16, dim=128, ff=8192, window=0),
    "4k": dict(width=4096, heads=32, dim=128, ff=16384, window=0),
    "8k": dict(width=8192, heads=64, dim=128, ff=32768, window=0),
}
FAMILIES = ("capped", "paired", "sigmoid", "attention", "delta")


def zudarax_config(s, kind):
    from petals_amd.models.zudarax.config import ZudaraxConfig

    rot = {"base": 10000.0, "dims": s["dim"]}
    mixer = {"heads": s["heads"], "kv_heads": s["heads"], "dim": s["dim"], "vdim": s["dim"], "rot": rot,
             "scale": s["dim"] ** -0.5}
    if kind == "capped":
        name = "attention"
        mixer.update(conv=4, softcap=50.0, mask={"size": 8192})
    elif kind == "paired":
        name = "attention_2"
        mixer.update(heads=s["heads"] // 2, kv_heads=s["heads"] // 2, vdim=2 * s["dim"], diff=0.5)
    else:
        name = "attention_3"
        mixer.update(conv=4, rot={**rot, "scaling": {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}})
    layer = {"type": name, "mixer": mixer, "mlp": {"kind": "dense", "ff": s["ff"]}}
    return ZudaraxConfig.from_hf_dict(
        {"layers": [layer] * LAYERS, "norm": {"eps": 1e-6, "groups": 2}, "vocab": 1024, "width": s["width"]},
        name_or_path="bench",
    )


def config_of(s, family):
    return lefulorn_config(s, family) if family in ("attention", "delta") else zudarax_config(s, family)


@torch.inference_mode()
def main(steps: int = 20, warmup: int = 5, sizes=None, families=FAMILIES, batches=(1, 8)):
    device = torch.device("cuda", 0)
    for name in sizes or SIZES:
        s = SIZES[name]
        for batch in batches:
            row = {"size": name, "layers": LAYERS, "batch": batch, "prefill_tokens": PREFILL, "context": CONTEXT}
            for f in families:  # in turn, on the same box
                prefill, decode = engine_runs(config_of(s, f), device, batch)
                if batch == 1:
                    row[f"{f}_prefill_tok_s"] = round(PREFILL / timed(prefill, max(3, steps // 4), 2))
                t = timed(decode, steps, warmup)
                row[f"{f}_decode_tok_s"] = round(batch / t)
                row[f"{f}_decode_us_per_layer"] = round(1e6 * t / LAYERS, 1)
                del prefill, decode
                torch.cuda.empty_cache()
            print(json.dumps(row), flush=True)


if __name__ == "__main__":
    import sys

    main(
        sizes=[a for a in sys.argv[1:] if a in SIZES] or None,
        families=tuple(a for a in sys.argv[1:] if a in FAMILIES) or FAMILIES,
        batches=tuple(int(a) for a in sys.argv[1:] if a.isdigit()) or (1, 8),
    )
