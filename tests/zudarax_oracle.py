"""Plain, slow oracle of the Zudarax design, written from its equations.

One function per mechanism, float64 throughout, whole sequences only: no cache,
no state that outlives a call, no batching, nothing imported from the framework.
Weights come as a dict of tensors under their checkpoint names. Attention is a
dense matrix of weights over all pairs, to be read against its formula.

``faults`` plants a mistake on purpose (tests use it to show that their inputs
would expose one); the names are at the places where they act.
"""

from __future__ import annotations

import json
import math
import os
from typing import Dict, FrozenSet, List, Optional

import torch

F64 = torch.float64
NONE: FrozenSet[str] = frozenset()


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def group_norm(x, w, groups, eps, faults=NONE):
    """Consecutive equal parts of the last axis, each by its own root mean square; one weight per value."""
    if "one_norm_group" in faults:
        groups = 1
    return rms(x.reshape(*x.shape[:-1], groups, -1), eps).reshape(x.shape) * w


# ------------------------------------------------------ ahead of the scores


def short_conv(u, w, faults=NONE):
    """u [S, C], w [C, taps]: y[t] = sum_j w[:, j] u[t - taps + 1 + j], zeros before the start."""
    taps = w.shape[1]
    if "no_conv" in faults:
        return u
    y = torch.zeros_like(u)
    for t in range(u.shape[0]):
        for j in range(taps):
            src = t - taps + 1 + j
            if "conv_one_less" in faults and j == 0 and taps > 1:
                continue
            if "conv_forgets" in faults and src < t // 2 * 2:  # inputs of earlier steps of two tokens
                continue
            if src >= 0:
                y[t] = y[t] + w[:, taps - 1 - j if "conv_reversed" in faults else j] * u[src]
    return y


def frequencies(rot, faults=NONE):
    """(radians per position of each pair, factor of cos and sin)"""
    dims, base, y = rot["dims"], rot["base"], rot.get("scaling")
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if y is None or "no_yarn" in faults:
        return f, 1.0

    def dim(turns):
        return dims * math.log(y["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo, hi = max(math.floor(dim(y["fast"])), 0), min(math.ceil(dim(y["slow"])), dims - 1)
    out = []
    for i, x in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(x / y["factor"] * ramp + x * (1.0 - ramp))
    return out, 1.0 if "no_yarn_factor" in faults else 0.1 * math.log(y["factor"]) + 1.0


def rotate(x, positions, rot, faults=NONE):
    """x [S, ..., n]: pairs (i, i + dims/2) of the first `dims` turned by position * frequency i."""
    half = rot["dims"] // 2
    freqs, factor = frequencies(rot, faults)
    if "no_rotation" in faults:
        return x
    out = list(x.unbind(-1))
    for i in range(half):
        angle = positions.to(F64) * freqs[i]
        angle = angle.view(-1, *[1] * (x.dim() - 2))
        i, j = (2 * i, 2 * i + 1) if "rotate_neighbours" in faults else (i, i + half)
        out[i] = (x[..., i] * torch.cos(angle) - x[..., j] * torch.sin(angle)) * factor
        out[j] = (x[..., j] * torch.cos(angle) + x[..., i] * torch.sin(angle)) * factor
    return torch.stack(out, dim=-1)


# ------------------------------------------------------------------- scores


def cap(score, limit):
    return limit * torch.tanh(score / limit)


def causal(s, faults=NONE):
    i, j = torch.arange(s)[:, None], torch.arange(s)[None, :]
    seen = j <= i
    if "forgets_far" in faults:
        seen = seen & (i - j < 64)
    return seen


def same_chunk(s, size, faults=NONE):
    i, j = torch.arange(s)[:, None], torch.arange(s)[None, :]
    if "chunk_slides" in faults:
        return (j <= i) & (i - j < size)
    off = 1 if "chunk_one_off" in faults else 0
    return (j <= i) & ((i + off) // size == (j + off) // size)


def softmax_weights(score, seen):
    return torch.softmax(score.masked_fill(~seen, -math.inf), dim=-1)


def sigmoid_weights(score, seen, bias, faults=NONE):
    """Every key for itself: nothing is divided by a sum over keys."""
    if "no_score_bias" in faults:
        bias = 0.0
    p = torch.where(seen, 1.0 / (1.0 + torch.exp(-(score + bias))), torch.zeros((), dtype=score.dtype))
    return p / p.sum(-1, keepdim=True) if "normalized" in faults else p


# ------------------------------------------------------------------- mixers


def capped_attention(h, w, m, eps, faults=NONE):
    """Softmax over a chunk with capped scores; biased projections, convolutions, norms of
    whole projections. h [S, width]; w: the mixer's tensors without their prefix; m: its config."""
    heads, kv, dim, vdim, s = m["heads"], m["kv_heads"], m["dim"], m["vdim"], h.shape[0]
    x = {}
    for n in "qkv":
        u = h @ w[n].T + (0.0 if "no_bias" in faults else w[n + ".b"])
        x[n] = short_conv(u, w[n + ".conv"], faults)
    for n, count in (("q", heads), ("k", kv)):
        if "norm_per_head" in faults:
            x[n] = rms(x[n].view(s, count, dim), eps).reshape(s, -1) * w[n + ".norm"]
        elif "no_qk_norm" not in faults:
            x[n] = rms(x[n], eps) * w[n + ".norm"]
        x[n] = rotate(x[n].view(s, count, dim), torch.arange(s), m["rot"], faults)
    v, out = x["v"].view(s, kv, vdim), []
    for a in range(heads):
        g = a // (heads // kv)
        score = x["q"][:, a] @ x["k"][:, g].T * m["scale"]
        if "no_cap" not in faults:
            score = cap(score, m["softcap"])
        out.append(softmax_weights(score, same_chunk(s, m["mask"]["size"], faults)) @ v[:, g])
    return torch.cat(out, dim=1) @ w["o"].T


def share_of_second_map(w, diff, faults=NONE):
    first, second = torch.exp((w["lq1"] * w["lk1"]).sum()), torch.exp((w["lq2"] * w["lk2"]).sum())
    return diff if "lambda_constant" in faults else first - second + diff


def paired_attention(h, w, m, eps, faults=NONE):
    """Differential attention: the difference of two softmax maps over the same values,
    normed, with a gate per head."""
    heads, kv, dim, vdim, s = m["heads"], m["kv_heads"], m["dim"], m["vdim"], h.shape[0]
    pos = torch.arange(s)
    q, k = ((h @ w[n].T).view(s, count, 2, dim) for n, count in (("q", heads), ("k", kv)))
    if "maps_outside" in faults:  # [map, head] instead of [head, map]
        q, k = (t.reshape(s, 2, -1, dim).transpose(1, 2) for t in (q, k))
    q, k = rotate(q, pos, m["rot"], faults), rotate(k, pos, m["rot"], faults)
    v = (h @ w["v"].T).view(s, kv, vdim)
    share, gate, out = share_of_second_map(w, m["diff"], faults), torch.sigmoid(h @ w["g"].T), []
    for a in range(heads):
        g = a // (heads // kv)
        one, two = (
            softmax_weights(q[:, a, n] @ k[:, g, n].T * m["scale"], causal(s, faults)) @ v[:, g] for n in (0, 1)
        )
        o = one if "one_map" in faults else one - share * two
        if "no_map_norm" not in faults:
            o = rms(o, eps)
        o = o * (1.0 if "no_map_factor" in faults else 1.0 - m["diff"])
        out.append(o if "no_gate" in faults else o * gate[:, a : a + 1])
    return torch.cat(out, dim=1) @ w["o"].T


def sigmoid_attention(h, w, m, eps, faults=NONE):
    """Sigmoid weights with a bias per head; convolutions; scaled frequencies."""
    heads, kv, dim, vdim, s = m["heads"], m["kv_heads"], m["dim"], m["vdim"], h.shape[0]
    q, k, v = (short_conv(h @ w[n].T, w[n + ".conv"], faults) for n in "qkv")
    q, k = (rotate(t.view(s, count, dim), torch.arange(s), m["rot"], faults) for t, count in ((q, heads), (k, kv)))
    v, out = v.view(s, kv, vdim), []
    for a in range(heads):
        g = a // (heads // kv)
        score = q[:, a] @ k[:, g].T * m["scale"]
        out.append(sigmoid_weights(score, causal(s, faults), w["pb"][a], faults) @ v[:, g])
    return torch.cat(out, dim=1) @ w["o"].T


MIXERS = {"attention": capped_attention, "attention_2": paired_attention, "attention_3": sigmoid_attention}


# ------------------------------------------------------------- feed-forward


def poly_norm(z, act, eps, faults=NONE):
    """Sum of the normed first three powers, and a constant."""
    a, b, c, e = act
    if "no_constant" in faults:
        e = 0.0
    if "powers_of_norm" in faults:
        n = rms(z, eps)
        return a * n + b * n**2 + c * n**3 + e
    return a * rms(z, eps) + b * rms(z**2, eps) + c * rms(z**3, eps) + e


def dense(h, w, eps, faults=NONE):
    """w: the feed-forward's tensors without their prefix."""
    return poly_norm(h @ w["up"].T, w["act"], eps, faults) @ w["down"].T


# -------------------------------------------------------------------- model


def run(
    config: dict,
    weights: Dict[str, torch.Tensor],
    tokens: List[int],
    *,
    faults: FrozenSet[str] = NONE,
    residuals: Optional[list] = None,
    embeds: Optional[torch.Tensor] = None,
) -> torch.Tensor:
    """Logits [S, vocab] of one sequence; `residuals` collects x after every layer."""
    weights = {k: v.to(F64) for k, v in weights.items()}
    eps, groups = config["norm"]["eps"], config["norm"]["groups"]
    x = weights["embed"][torch.as_tensor(tokens)] if embeds is None else embeds.to(F64)
    for i, layer in enumerate(config["layers"]):
        p = f"l{i}."
        mix, mlp = ({k[len(p) + 4 :]: t for k, t in weights.items() if k.startswith(p + part)} for part in ("mix.", "mlp."))
        h = group_norm(x, weights[p + "norm1"], groups, eps, faults)
        add = MIXERS[layer["type"]](h, mix, layer["mixer"], eps, faults)
        if "in_turn" in faults:
            x, add = x + add, 0.0
            h = group_norm(x, weights[p + "norm1"], groups, eps, faults)
        if layer.get("mlp") is not None:
            add = add + dense(h, mlp, eps, faults)
        x = x + add
        if residuals is not None:
            residuals.append(x.clone())
    return group_norm(x, weights["final.norm"], groups, eps, faults) @ weights["head"].T


# ------------------------------------------------------- random small models


def random_model(config: dict, seed: int = 0) -> Dict[str, torch.Tensor]:
    """bf16 checkpoint tensors of `config` (row scale ~ 1/sqrt(in), vectors off their neutral value)."""
    gen = torch.Generator().manual_seed(seed)

    def mat(out, inp, gain=1.0):
        return (torch.randn(out, inp, generator=gen) * (gain / math.sqrt(inp))).to(torch.bfloat16)

    def vec(n, center, spread=0.3):
        return (center + spread * torch.randn(n, generator=gen)).to(torch.bfloat16)

    d = config["width"]
    w = {"embed": torch.randn(config["vocab"], d, generator=gen).to(torch.bfloat16),
         "head": mat(config["vocab"], d, 2.0), "final.norm": vec(d, 1.0)}
    for i, layer in enumerate(config["layers"]):
        m, p, kind = layer["mixer"], f"l{i}.mix.", layer["type"]
        heads, kv, maps = m["heads"], m["kv_heads"], 2 if kind == "attention_2" else 1
        rows = {"q": heads * maps * m["dim"], "k": kv * maps * m["dim"], "v": kv * m["vdim"]}
        w[f"l{i}.norm1"] = vec(d, 1.0)
        for n, r in rows.items():
            w[p + n] = mat(r, d, 1.0 if n == "v" else 1.5)
            if kind == "attention":
                w[p + n + ".b"] = vec(r, 0.0, 0.5)
            if kind != "attention_2":
                w[p + n + ".conv"] = mat(r, m["conv"], 1.3)
        w[p + "o"] = mat(d, heads * m["vdim"])
        if kind == "attention":
            w[p + "q.norm"], w[p + "k.norm"] = vec(rows["q"], 1.2), vec(rows["k"], 1.2)
        elif kind == "attention_2":
            for n in ("lq1", "lk1", "lq2", "lk2"):
                w[p + n] = vec(m["dim"], 0.1, 0.3 / math.sqrt(m["dim"]) + 0.1)
            w[p + "g"] = mat(heads, d, 2.0)
        else:
            w[p + "pb"] = vec(heads, -2.5, 0.5)
        if layer.get("mlp") is not None:
            ff = layer["mlp"]["ff"]
            w[f"l{i}.mlp.up"], w[f"l{i}.mlp.down"] = mat(ff, d), mat(d, ff)
            w[f"l{i}.mlp.act"] = vec(4, 0.5, 0.3)
    return w


def config_dict(vocab=97, width=40, eps=1e-6, groups=2, layers=()) -> dict:
    return {"architecture": "Zudarax", "layers": [dict(l) for l in layers], "norm": {"eps": eps, "groups": groups},
            "vocab": vocab, "width": width}


def _layer(kind, ff, mixer) -> dict:
    return {"type": kind, "mlp": None if ff is None else {"ff": ff, "kind": "dense"}, "mixer": mixer}


def capped_layer(heads=4, kv_heads=2, dim=16, vdim=12, conv=3, size=50, rot=8, base=300.0, scale=0.3, softcap=3.0,
                 ff=56) -> dict:
    return _layer("attention", ff, {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "mask": {"size": size},
        "rot": {"base": base, "dims": rot}, "scale": scale, "softcap": softcap,
    })


def paired_layer(heads=4, kv_heads=2, dim=12, vdim=20, rot=6, base=900.0, scale=0.35, diff=0.6, ff=None) -> dict:
    return _layer("attention_2", ff, {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "rot": {"base": base, "dims": rot},
        "scale": scale, "diff": diff,
    })


def sigmoid_layer(heads=6, kv_heads=3, dim=14, vdim=10, conv=4, rot=12, base=5000.0, scale=0.3, factor=6.0, original=90,
                  fast=10.0, slow=0.5, ff=30) -> dict:
    return _layer("attention_3", ff, {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv,
        "rot": {"base": base, "dims": rot,
                "scaling": {"factor": factor, "original": original, "fast": fast, "slow": slow}},
        "scale": scale,
    })


def save_model(path, config: dict, weights: Dict[str, torch.Tensor]) -> None:
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(config, f)
    save_file({k: v.contiguous() for k, v in weights.items()}, os.path.join(path, "model.safetensors"))
