"""Plain, slow oracle of the Lefulorn design, written from its equations.

One function per mechanism, float64 throughout, whole sequences only: no cache,
no state that outlives a call, no batching, nothing imported from the framework.
Weights come as a dict of tensors under their checkpoint names. Windows are
dense masks and the recurrence is a loop over tokens, to be read against their
formulas.

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


def norm(x, w, eps):
    return rms(x, eps) * w


def silu(x):
    return x / (1.0 + torch.exp(-x))


# ------------------------------------------------------------ channel_delta


def short_conv(x, w, faults=NONE):
    """x [S, C], w [C, taps]: y[t] = sum_j w[:, j] x[t - (taps - 1) + j], zeros before the start."""
    taps = w.shape[1]
    y = torch.zeros_like(x)
    for t in range(x.shape[0]):
        for j in range(taps):
            src = t - (taps - 1) + j
            if "conv_reversed" in faults:
                src = t - j
            if "conv_one_less" in faults and j == 0 and taps > 1:
                continue
            if src >= 0:
                y[t] = y[t] + w[:, j] * x[src]
    return y


def unit(x):
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + 1e-6)


def channel_decay(h, w_a1, w_a2, a_log, dt_bias, heads, dim):
    """g [S, heads, dim] in (0, 1)."""
    a = (h @ w_a1.T) @ w_a2.T + dt_bias
    softplus = torch.log1p(torch.exp(-a.abs())) + a.clamp(min=0)
    return torch.exp(-torch.exp(a_log)[None, :, None] * softplus.view(-1, heads, dim))


def delta_rule(q, k, v, g, beta, faults=NONE):
    """q, k, g [S, H, dim], v [S, H, vdim], beta [S, H] -> o [S, H, vdim]."""
    s, heads, dim = q.shape
    state = torch.zeros(heads, dim, v.shape[-1], dtype=q.dtype)
    out = []
    for t in range(s):
        read = state
        if "decay_after" not in faults:
            state = g[t][:, :, None] * state
        u = beta[t][:, None] * (v[t] - (k[t][:, :, None] * state).sum(1))
        if "no_delta" in faults:
            u = beta[t][:, None] * v[t]
        state = state + k[t][:, :, None] * u[:, None, :]
        if "decay_after" in faults:
            state = g[t][:, :, None] * state
        if "read_before_write" not in faults:
            read = state
        out.append((q[t][:, :, None] * read).sum(1))
    return torch.stack(out)


def channel_delta(h, w, m, eps, faults=NONE):
    """h [S, width]; w: the mixer's tensors without their prefix; m: its config."""
    heads, kv, dim, vdim = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"]
    s = h.shape[0]
    q, k, v = (silu(short_conv(h @ w[n].T, w[n + ".conv"], faults)) for n in ("q", "k", "v"))
    q, k = unit(q.view(s, kv, dim)) * dim**-0.5, unit(k.view(s, kv, dim))
    of = torch.arange(heads) // (heads // kv)
    if "head_interleave" in faults:
        of = torch.arange(heads) % kv
    q, k = q[:, of], k[:, of]
    beta = torch.sigmoid(h @ w["b"].T)
    g = channel_decay(h, w["a1"], w["a2"], w["A_log"], w["dt_bias"], heads, dim)
    o = delta_rule(q, k, v.view(s, heads, vdim), g, beta, faults)
    gate = torch.sigmoid((h @ w["g1"].T) @ w["g2"].T).view(s, heads, vdim)
    return (norm(o, w["norm"], eps) * gate).reshape(s, heads * vdim) @ w["o"].T


# ---------------------------------------------------------------- attention


def temperature(positions, coef, every):
    return 1.0 + coef * torch.log(torch.floor((positions + 1.0) / every) + 1.0)


def window_mask(s: int, size: int, faults=NONE) -> torch.Tensor:
    """visible[i, j] iff 0 <= i - j < size."""
    size += ("window+1" in faults) - ("window-1" in faults)
    gap = torch.arange(s)[:, None] - torch.arange(s)[None, :]
    return (gap >= 0) & (gap < size)


def sink_softmax(score, sink, faults=NONE):
    """score [S, S] with -inf where nothing is seen; sink: one more entry of the denominator."""
    if "no_sink" in faults:
        return torch.softmax(score, dim=-1)
    top = torch.maximum(score.max(dim=-1, keepdim=True).values, sink)
    e = torch.exp(score - top)
    return e / (e.sum(dim=-1, keepdim=True) + torch.exp(sink - top))


def slope(head, heads):
    return 2.0 ** (-8.0 * (head + 1) / heads)


def attention(h, w, m, first: Optional[torch.Tensor], faults=NONE):
    """Returns (output [S, width], this layer's own values [S, G * vdim]).
    first: the values of the first mixing layer, None where nothing is mixed."""
    heads, kv, dim, vdim = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"]
    s = h.shape[0]
    q, k, v = (h @ w[n].T + w[n + ".b"] for n in ("q", "k", "v"))
    own = v
    if first is not None and "no_mix" not in faults:
        v = (1.0 - w["vmix"]) * v + w["vmix"] * first
    q, k, v = q.view(s, heads, dim), k.view(s, kv, dim), v.view(s, kv, vdim)
    pos = torch.arange(s)
    if "no_temp" not in faults:
        q = q * temperature(pos.to(F64), m["q_temp"]["coef"], m["q_temp"]["every"] + ("temp_edge" in faults))[:, None, None]
    seen = window_mask(s, m["mask"]["size"], faults)
    gap = (pos[:, None] - pos[None, :]).to(F64)
    out = torch.zeros(s, heads, vdim, dtype=h.dtype)
    for n in range(heads):
        of = n // (heads // kv)
        score = (q[:, n] @ k[:, of].T) * m["scale"]
        if "no_bias" not in faults:
            score = score - slope(n, heads) * (gap if "key_bias" not in faults else -pos[None, :].to(F64))
        score = score.masked_fill(~seen, -math.inf)
        out[:, n] = sink_softmax(score, w["sink"][n], faults) @ v[:, of]
    y = out.reshape(s, heads * vdim)
    if "no_gate" not in faults:
        y = y * torch.sigmoid(h @ w["g"].T)
    return y @ w["o"].T, own


# ------------------------------------------------------------- feed-forward


def dense(h, w, faults=NONE):
    """w: the feed-forward's tensors without their prefix."""
    a = torch.relu(h @ w["up"].T + w["up.b"])
    return (a if "no_square" in faults else a * a) @ w["down"].T + w["down.b"]


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
    eps = config["norm"]["eps"]
    x = weights["embed"][torch.as_tensor(tokens)] if embeds is None else embeds.to(F64)
    first = None
    for i, layer in enumerate(config["layers"]):
        m, p = layer["mixer"], f"l{i}."
        w = {k[len(p) + 4 :]: t for k, t in weights.items() if k.startswith(p + "mix.")}
        h = norm(x, weights[p + "norm1"], eps)
        if layer["type"] == "channel_delta":
            x = x + channel_delta(h, w, m, eps, faults)
        else:
            mixes = bool(m.get("v_mix"))
            y, own = attention(h, w, m, first if mixes else None, faults)
            if mixes and (first is None or "mix_with_last" in faults):
                first = own
            x = x + y
        if layer.get("mlp") is not None:
            w = {k[len(p) + 4 :]: t for k, t in weights.items() if k.startswith(p + "mlp.")}
            x = x + dense(norm(x, weights[p + "norm2"], eps), w, faults)
        if residuals is not None:
            residuals.append(x.clone())
    return norm(x, weights["final.norm"], eps) @ weights["head"].T * config["logit_scale"]


# ------------------------------------------------------- random small models


def random_model(config: dict, seed: int = 0, rank: int = 6, gate_rank: int = 5) -> Dict[str, torch.Tensor]:
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
        m, p = layer["mixer"], f"l{i}."
        heads, dim, vdim = m["heads"], m["dim"], m["vdim"]
        kv = m.get("kv_heads", heads)
        w[p + "norm1"] = vec(d, 1.0)
        p += "mix."
        w[p + "o"] = mat(d, heads * vdim)
        if layer["type"] == "channel_delta":
            for name, n in (("q", kv * dim), ("k", kv * dim), ("v", heads * vdim)):
                w[p + name] = mat(n, d)
                w[p + name + ".conv"] = mat(n, m["conv"], 1.5)
            w[p + "b"] = mat(heads, d)
            w[p + "A_log"] = vec(heads, -1.5, 1.0)
            w[p + "dt_bias"] = vec(heads * dim, -1.0, 1.0)
            w[p + "a1"], w[p + "a2"] = mat(rank, d), mat(heads * dim, rank)
            w[p + "g1"], w[p + "g2"] = mat(gate_rank, d), mat(heads * vdim, gate_rank, 2.0)
            w[p + "norm"] = vec(vdim, 1.0)
        else:
            for name, n, gain in (("q", heads * dim, 2.0), ("k", kv * dim, 2.0), ("v", kv * vdim, 1.0)):
                w[p + name] = mat(n, d, gain)
                w[p + name + ".b"] = vec(n, 0.0)
            if m.get("v_mix"):
                w[p + "vmix"] = vec(1, 0.6, 0.1)[0].clone()
            w[p + "sink"] = vec(heads, 0.5, 1.0)
            w[p + "g"] = mat(heads * vdim, d)
        if layer.get("mlp") is not None:
            p = f"l{i}."
            ff = layer["mlp"]["ff"]
            w[p + "norm2"] = vec(d, 1.0)
            w[p + "mlp.up"], w[p + "mlp.up.b"] = mat(ff, d), vec(ff, 0.0)
            w[p + "mlp.down"], w[p + "mlp.down.b"] = mat(d, ff), vec(d, 0.0)
    return w


def config_dict(vocab=97, width=40, eps=1e-6, logit_scale=0.7, layers=()) -> dict:
    return {"architecture": "Lefulorn", "layers": [dict(l) for l in layers], "logit_scale": logit_scale,
            "norm": {"eps": eps}, "vocab": vocab, "width": width}


def _ff(ff) -> Optional[dict]:
    return None if ff is None else {"ff": ff, "kind": "dense"}


def delta_layer(heads=4, kv_heads=2, dim=12, vdim=20, conv=4, ff=None) -> dict:
    return {"type": "channel_delta", "mlp": _ff(ff),
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def attention_layer(heads=6, kv_heads=2, dim=16, vdim=12, window=20, coef=0.3, every=11, scale=0.2, v_mix=True,
                    ff=56) -> dict:
    return {"type": "attention", "mlp": _ff(ff),
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window},
                      "q_temp": {"coef": coef, "every": every}, "scale": scale, "v_mix": v_mix}}


def save_model(path, config: dict, weights: Dict[str, torch.Tensor]) -> None:
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(config, f)
    save_file({k: v.contiguous() for k, v in weights.items()}, os.path.join(path, "model.safetensors"))
