"""Prefill and decode throughput of Soselix layers beside layers of equal size of the
closest families, random weights, one GPU.

Run through `bench.py --compare soselix`. Each side runs a stack of equal layers with
the span engine that serves it (decode: its captured graph):

  hgrn2, mamba2, latent   the three mixers, each with a feed-forward of 4x width
  delta, attention        Lefulorn's two mixers with the same feed-forward (pre-norm,
                          32-bit residual; attention over all earlier tokens here)
  latent_only             latent attention without a feed-forward, and
  tulezen                 Tulezen's, likewise, over all earlier tokens

Prints one JSON line per size and batch.
"""

from __future__ import annotations

import json

import torch

from benchmarks.benchmark_lefulorn import CONTEXT, LAYERS, PREFILL, engine_runs, lefulorn_config
from benchmarks.benchmark_tulezen import timed

SIZES = {
    "2k": dict(width=2048, heads=16, dim=128, ff=8192, window=0, q_rank=768),
    "4k": dict(width=4096, heads=32, dim=128, ff=16384, window=0, q_rank=1536),
    "8k": dict(width=8192, heads=64, dim=128, ff=32768, window=0, q_rank=3072),
}
KV_RANK, ROT, STATE, GROUPS = 512, 64, 128, 8
FAMILIES = ("hgrn2", "mamba2", "delta", "latent", "attention", "latent_only", "tulezen")


def soselix_config(s, kind):
    from petals_amd.models.soselix.config import SoselixConfig

    if kind == "hgrn2":
        layer = {"type": kind, "mixer": {"heads": s["heads"], "dim": s["dim"], "vdim": s["dim"]}}
    elif kind == "mamba2":
        layer = {"type": kind, "mixer": {
            "heads": 2 * s["width"] // 64, "vdim": 64, "state": STATE, "groups": GROUPS, "norm_groups": GROUPS, "conv": 4,
        }}
    else:
        layer = {"type": "latent_attention", "mixer": {
            "heads": s["heads"], "dim": s["dim"], "vdim": s["dim"], "rot_dim": ROT, "kv_rank": KV_RANK,
            "q_rank": s["q_rank"], "rot": {"base": 10000.0, "dims": ROT}, "scale": (s["dim"] + ROT) ** -0.5,
        }}
    layer["mlp"] = None if kind == "latent_only" else {"kind": "dense", "ff": s["ff"]}
    return SoselixConfig.from_hf_dict(
        {"layers": [layer] * LAYERS, "norm": {"eps": 1e-6}, "vocab": 1024, "width": s["width"], "residual_mult": 0.5},
        name_or_path="bench",
    )


def tulezen_config(s):
    from petals_amd.models.tulezen.config import TulezenConfig

    layer = {"type": "latent_attention", "mixer": {
        "heads": s["heads"], "dim": s["dim"], "vdim": s["dim"], "kv_rank": KV_RANK, "scale": s["dim"] ** -0.5,
    }, "mlp": None}
    return TulezenConfig.from_hf_dict(
        {"layers": [layer] * LAYERS, "norm": {"eps": 1e-6}, "vocab": 1024, "width": s["width"]}, name_or_path="bench"
    )


def config_of(s, family):
    if family == "tulezen":
        return tulezen_config(s)
    return lefulorn_config(s, family) if family in ("delta", "attention") else soselix_config(s, family)


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
