"""Plain, slow oracle of the Tulezen design, written from its equations.

One function per mechanism, float64 throughout, whole sequences only: no cache,
no pages, no batching, nothing imported from the framework. Weights come as a
dict of tensors under their checkpoint names. Windows and expert selection are
spelled out as dense masks and loops, to be read against their formulas.

``faults`` plants a mistake on purpose (tests use it to show that their inputs
would expose one): "window+1", "window-1", "no_share", "renorm_router",
"no_plus_one", "no_limit", "plain_norm".
"""

from __future__ import annotations

import math
from typing import Dict, FrozenSet, List, Optional

import torch

F64 = torch.float64


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def zero_centered_norm(x, w, eps, faults: FrozenSet[str] = frozenset()):
    return rms(x, eps) * (w if "plain_norm" in faults else 1.0 + w)


def latent(h, w_dkv, w_norm, eps):
    """c [S, R]: the normalised down-projection that a cache would hold."""
    return rms(h @ w_dkv.T, eps) * w_norm


def window_mask(s: int, size: int, faults: FrozenSet[str] = frozenset()) -> torch.Tensor:
    """visible[i, j] iff 0 <= i - j < size."""
    if "window+1" in faults:
        size += 1
    if "window-1" in faults:
        size -= 1
    i = torch.arange(s)[:, None]
    j = torch.arange(s)[None, :]
    return (i - j >= 0) & (i - j < size)


def latent_attention(h, c, w_q, w_uk, w_uv, w_o, *, heads, dim, vdim, scale, window, faults=frozenset()):
    """Position-free attention whose keys and values are projections of c."""
    s = h.shape[0]
    q = (h @ w_q.T).view(s, heads, dim)
    k = (c @ w_uk.T).view(s, heads, dim)
    v = (c @ w_uv.T).view(s, heads, vdim)
    visible = window_mask(s, window, faults)
    out = torch.zeros(s, heads, vdim, dtype=h.dtype)
    for n in range(heads):
        score = (q[:, n] @ k[:, n].T) * scale
        score = score.masked_fill(~visible, -math.inf)
        out[:, n] = torch.softmax(score, dim=-1) @ v[:, n]
    return out.reshape(s, heads * vdim) @ w_o.T


def expert(h, w_gate, w_up, w_down, limit, faults=frozenset()):
    g, u = h @ w_gate.T, h @ w_up.T
    if "no_limit" not in faults:
        g = torch.clamp(g, max=limit)
        u = torch.clamp(u, min=-limit, max=limit)
    y = g * torch.sigmoid(1.702 * g) * (u if "no_plus_one" in faults else u + 1.0)
    return y @ w_down.T


def route(h, w_router, top, faults=frozenset()):
    """(weights [S, top], experts [S, top]): softmax over all, no renormalisation."""
    p = torch.softmax(h @ w_router.T, dim=-1)
    w, e = torch.topk(p, top, dim=-1)
    if "renorm_router" in faults:
        w = w / w.sum(-1, keepdim=True)
    return w, e


def moe(h, weights: Dict[str, torch.Tensor], prefix: str, *, experts, top, limit, faults=frozenset()):
    w, chosen = route(h, weights[prefix + "router"], top, faults)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for slot in range(top):
            e = f"{prefix}e{int(chosen[t, slot])}."
            out[t] += w[t, slot] * expert(
                h[t], weights[e + "gate"], weights[e + "up"], weights[e + "down"], limit, faults
            )
    return out


def run(
    config: dict,
    weights: Dict[str, torch.Tensor],
    tokens: List[int],
    *,
    faults: FrozenSet[str] = frozenset(),
    residuals: Optional[list] = None,
    embeds: Optional[torch.Tensor] = None,
) -> torch.Tensor:
    """Logits [S, vocab] of one sequence; `residuals` collects x after every layer."""
    weights = {k: v.to(F64) for k, v in weights.items()}
    eps = config["norm"]["eps"]
    x = weights["embed"][torch.as_tensor(tokens)] if embeds is None else embeds.to(F64)
    latents = {}
    for i, layer in enumerate(config["layers"]):
        m, p = layer["mixer"], f"l{i}."
        src = m.get("kv_from")
        if src is None or ("no_share" in faults and src is not None):
            own = i if src is None else src
            latents[i] = latent(x, weights[f"l{own}.mix.dkv"], weights[f"l{own}.mix.dkv.norm"], eps)
            c = latents[i]
        else:
            c = latents[src]
        y = latent_attention(
            x, c, weights[p + "mix.q"], weights[p + "mix.uk"], weights[p + "mix.uv"], weights[p + "mix.o"],
            heads=m["heads"], dim=m["dim"], vdim=m["vdim"], scale=m["scale"], window=m["mask"]["size"],
            faults=faults,
        )
        x = x + zero_centered_norm(y, weights[p + "norm1"], eps, faults)
        if layer.get("mlp") is not None:
            f = layer["mlp"]
            y = moe(x, weights, p + "mlp.", experts=f["router"]["experts"], top=f["router"]["top"],
                    limit=f["expert"]["limit"], faults=faults)
            x = x + zero_centered_norm(y, weights[p + "norm2"], eps, faults)
        if residuals is not None:
            residuals.append(x.clone())
    return zero_centered_norm(x, weights["final.norm"], eps, faults) @ weights["head"].T


def random_model(config: dict, seed: int = 0, scale: float = 1.0, decided: bool = False) -> Dict[str, torch.Tensor]:
    """bf16 checkpoint tensors of `config` (row scale ~ 1/sqrt(in), norms off their neutral value).

    decided: the routers read a few dimensions that no sublayer adds to (their
    norm weights are -1), so that each token's experts are fixed by its embedding
    and 16-bit rounding cannot turn a close call into another expert."""
    g = torch.Generator().manual_seed(seed)

    def mat(out, inp, gain=1.0):
        return (torch.randn(out, inp, generator=g) * (gain * scale / math.sqrt(inp))).to(torch.bfloat16)

    def vec(n, center):
        return (center + 0.3 * torch.randn(n, generator=g)).to(torch.bfloat16)

    d = config["width"]
    fixed = max(2, d // 5)
    w = {"embed": torch.randn(config["vocab"], d, generator=g).to(torch.bfloat16),
         "head": mat(config["vocab"], d), "final.norm": vec(d, 0.0)}
    for i, layer in enumerate(config["layers"]):
        m, p = layer["mixer"], f"l{i}."
        h, dim, vdim, r = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
        w[p + "norm1"] = vec(d, 0.0)
        w[p + "mix.q"] = mat(h * dim, d, 2.0)
        if m.get("kv_from") is None:
            w[p + "mix.dkv"] = mat(r, d)
            w[p + "mix.dkv.norm"] = vec(r, 1.0)
        w[p + "mix.uk"] = mat(h * dim, r, 2.0)
        w[p + "mix.uv"] = mat(h * vdim, r)
        w[p + "mix.o"] = mat(d, h * vdim)
        if layer.get("mlp") is not None:
            w[p + "norm2"] = vec(d, 0.0)
            ff = layer["mlp"]["expert"]["ff"]
            n = layer["mlp"]["router"]["experts"]
            w[p + "mlp.router"] = mat(n, d, 2.0)
            if decided:
                w[p + "mlp.router"][:, fixed:] = 0
            for e in range(n):
                w[p + f"mlp.e{e}.gate"] = mat(ff, d, 2.0)
                w[p + f"mlp.e{e}.up"] = mat(ff, d, 2.0)
                w[p + f"mlp.e{e}.down"] = mat(d, ff)
        if decided:
            for norm in ("norm1", "norm2")[: 1 if layer.get("mlp") is None else 2]:
                w[p + norm][:fixed] = -1
    return w


def config_dict(vocab=97, width=40, eps=1e-6, layers=()) -> dict:
    return {"architecture": "Tulezen", "layers": [dict(l) for l in layers], "norm": {"eps": eps},
            "vocab": vocab, "width": width}


def layer_dict(heads=3, dim=16, vdim=24, kv_rank=32, window=20, scale=0.05, kv_from=None, ff=40, limit=1.5,
               experts=5, top=2, mlp=True) -> dict:
    mixer = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale, "mask": {"size": window}}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    ffd = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    return {"type": "latent_attention", "mixer": mixer, "mlp": ffd if mlp else None}


def save_model(path, config: dict, weights: Dict[str, torch.Tensor]) -> None:
    import json
    import os

    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(config, f)
    save_file({k: v.contiguous() for k, v in weights.items()}, os.path.join(path, "model.safetensors"))
