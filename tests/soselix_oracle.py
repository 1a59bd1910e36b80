"""Plain, slow oracle of the Soselix design, written from its equations.

One function per mechanism, float64 throughout, whole sequences only: no cache,
no state that outlives a call, no batching, nothing imported from the framework.
Weights come as a dict of tensors under their checkpoint names. Attention is a
dense masked softmax and the recurrences are loops over tokens, to be read
against their formulas.

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
    """w: one weight per coordinate, or a single number for all of them."""
    return rms(x, eps) * w


def silu(x):
    return x / (1.0 + torch.exp(-x))


def softplus(x):
    return torch.log1p(torch.exp(-x.abs())) + x.clamp(min=0)


# --------------------------------------------------------- latent attention


def rotate(x, positions, dims, base, faults=NONE):
    """x [S, ..., n]: pairs (i, i + dims/2) of the first `dims` turned by position * base^(-2i/dims)."""
    half = dims // 2
    if "no_rotation" in faults:
        return x
    out = list(x.unbind(-1))
    for i in range(half):
        angle = positions.to(F64) * base ** (-2.0 * i / dims)
        angle = angle.view(-1, *[1] * (x.dim() - 2))
        i, j = (2 * i, 2 * i + 1) if "rotate_neighbours" in faults else (i, i + half)
        out[i] = x[..., i] * torch.cos(angle) - x[..., j] * torch.sin(angle)
        out[j] = x[..., j] * torch.cos(angle) + x[..., i] * torch.sin(angle)
    return torch.stack(out, dim=-1)


def latent_rows(h, w, m, eps, faults=NONE):
    """(latent c [S, kv_rank], rotated shared key part [S, rot_dim])."""
    y = h @ w["dkv"].T
    c = norm(y[:, : m["kv_rank"]], w["dkv.norm"], eps)
    return c, rotate(y[:, m["kv_rank"] :], torch.arange(len(h)), m["rot"]["dims"], m["rot"]["base"], faults)


def sink_softmax(score, sink, faults=NONE):
    """score [S, S] with -inf where nothing is seen; sink: one more entry of the denominator."""
    if "no_sink" in faults:
        return torch.softmax(score, dim=-1)
    top = torch.maximum(score.max(dim=-1, keepdim=True).values, sink)
    e = torch.exp(score - top)
    return e / (e.sum(dim=-1, keepdim=True) + torch.exp(sink - top))


def latent_attention(h, w, m, eps, rows, faults=NONE):
    """rows: (latent, key part) of the layer whose cache is read."""
    heads, dim, rot, vdim = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    s = h.shape[0]
    c, shared = rows
    q = (norm(h @ w["dq"].T, w["dq.norm"], eps) @ w["uq"].T).view(s, heads, dim + rot)
    q_plain = q[:, :, :dim]
    q_turned = rotate(q[:, :, dim:], torch.arange(s), m["rot"]["dims"], m["rot"]["base"], faults)
    k, v = (c @ w["uk"].T).view(s, heads, dim), (c @ w["uv"].T).view(s, heads, vdim)
    gap = torch.arange(s)[:, None] - torch.arange(s)[None, :]
    seen = gap >= 0
    if "forgets_far" in faults:
        seen = seen & (gap < 64)
    out = []
    gate = torch.sigmoid(h @ w["g"].T)
    for n in range(heads):
        score = (q_plain[:, n] @ k[:, n].T + q_turned[:, n] @ shared.T) * m["scale"]
        score = score.masked_fill(~seen, -math.inf)
        o = sink_softmax(score, w["sink"][n], faults) @ v[:, n]
        out.append(o if "no_gate" in faults else o * gate[:, n : n + 1])
    return torch.cat(out, dim=1) @ w["o"].T


# -------------------------------------------------------------------- hgrn2


def forget_gate(z, lower):
    return lower + (1.0 - lower) / (1.0 + torch.exp(-z))


def decay_recurrence(q, k, v, f, faults=NONE):
    """q, k, f [S, H, dim], v [S, H, vdim] -> S^T q with S <- f S + k v^T, [S, H, vdim]."""
    state = torch.zeros(q.shape[1], q.shape[2], v.shape[2], dtype=q.dtype)
    out = []
    for t in range(q.shape[0]):
        read = state
        if "lost_state" in faults and t == q.shape[0] // 2:
            state = torch.zeros_like(state)
        state = f[t][:, :, None] * state + k[t][:, :, None] * v[t][:, None, :]
        if "read_before_write" not in faults:
            read = state
        out.append((q[t][:, :, None] * read).sum(1))
    return torch.stack(out)


def hgrn2(h, w, m, eps, faults=NONE):
    """h [S, width]; w: the mixer's tensors without their prefix; m: its config."""
    heads, dim, vdim = m["heads"], m["dim"], m["vdim"]
    s = h.shape[0]
    q, v = silu(h @ w["q"].T).view(s, heads, dim), (h @ w["v"].T).view(s, heads, vdim)
    lower = torch.zeros_like(w["lower"]) if "no_lower" in faults else w["lower"]
    f = forget_gate(h @ w["f"].T + w["f.b"], lower).view(s, heads, dim)
    k = torch.ones_like(f) if "write_all" in faults else 1.0 - f
    o = decay_recurrence(q, k, v, f, faults)
    return norm(o, w["norm"], eps).reshape(s, heads * vdim) @ w["o"].T


# ------------------------------------------------------------------- mamba2


def short_conv(x, w, bias, faults=NONE):
    """x [S, C], w [C, taps]: y[t] = bias + sum_j w[:, j] x[t - (taps - 1) + j], zeros before the start."""
    taps = w.shape[1]
    y = torch.zeros_like(x) + (0.0 if "no_conv_bias" in faults else bias)
    for t in range(x.shape[0]):
        for j in range(taps):
            src = t - (taps - 1) + j
            if "conv_one_less" in faults and j == 0 and taps > 1:
                continue
            if src >= 0:
                y[t] = y[t] + w[:, j] * x[src]
    return y


def group_norm(y, w, parts, eps):
    """Equal parts of the last axis, each by its own root mean square."""
    return rms(y.view(*y.shape[:-1], parts, -1), eps).reshape(y.shape) * w


def mamba2(h, w, m, eps, faults=NONE):
    heads, vdim, n, groups = m["heads"], m["vdim"], m["state"], m["groups"]
    inner, s = heads * vdim, h.shape[0]
    z, xbc, dt = (h @ w["in"].T).split([inner, inner + 2 * groups * n, heads], dim=-1)
    xbc = silu(short_conv(xbc, w["conv"], w["conv.b"], faults))
    x, b, c = xbc.split([inner, groups * n, groups * n], dim=-1)
    x = x.reshape(s, heads, vdim)
    of = torch.arange(heads) // (heads // groups)
    if "group_interleave" in faults:
        of = torch.arange(heads) % groups
    b, c = b.reshape(s, groups, n)[:, of], c.reshape(s, groups, n)[:, of]
    dt = softplus(dt + w["dt_bias"])
    if "dt_clamp" in faults:
        dt = dt.clamp(max=0.5)
    decay = torch.exp(-torch.exp(w["A_log"]) * dt)[:, :, None].expand(s, heads, n)
    y = decay_recurrence(c, b, dt[:, :, None] * x, decay, faults)
    if "no_skip" not in faults:
        y = y + w["D"][None, :, None] * x
    y = y.reshape(s, inner)
    if "gate_after" in faults:
        return (group_norm(y, w["norm"], m["norm_groups"], eps) * silu(z)) @ w["o"].T
    return group_norm(y * silu(z), w["norm"], 1 if "one_norm" in faults else m["norm_groups"], eps) @ w["o"].T


# ------------------------------------------------------------- feed-forward


def xielu(z, p, q, faults=NONE):
    positive = softplus(p) * z * z + 0.5 * z
    negative = (0.5 + softplus(q)) * (torch.expm1(z.clamp(max=0)) - z) + 0.5 * z
    if "act_half" in faults:
        negative = softplus(q) * (torch.expm1(z.clamp(max=0)) - z) + 0.5 * z
    return torch.where(z > 0, positive, negative)


def dense(h, w, faults=NONE):
    """w: the feed-forward's tensors without their prefix."""
    a = xielu(h @ w["up"].T + w["up.b"], w["act"][0], w["act"][1], faults)
    return a @ w["down"].T + w["down.b"]


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
    eps, mult = config["norm"]["eps"], config["residual_mult"]
    x = weights["embed"][torch.as_tensor(tokens)] * config["embedding"]["scale"] if embeds is None else embeds.to(F64)
    rows = {}
    for i, layer in enumerate(config["layers"]):
        m, p = layer["mixer"], f"l{i}."
        w = {k[len(p) + 4 :]: t for k, t in weights.items() if k.startswith(p + "mix.")}
        h = norm(x, weights[p + "norm1"], eps)
        if layer["type"] == "latent_attention":
            source = m.get("kv_from")
            if source is None:
                rows[i] = latent_rows(h, w, m, eps, faults)
            y = latent_attention(h, w, m, eps, rows[i if source is None else source], faults)
        else:
            y = (hgrn2 if layer["type"] == "hgrn2" else mamba2)(h, w, m, eps, faults)
        x = x + mult * y
        if layer.get("mlp") is not None:
            w = {k[len(p) + 4 :]: t for k, t in weights.items() if k.startswith(p + "mlp.")}
            x = x + mult * dense(norm(x, weights[p + "norm2"], eps), w, faults)
        if residuals is not None:
            residuals.append(x.clone())
    return norm(x, weights["final.norm"], eps) @ weights["head"].T


# ------------------------------------------------------- random small models


def random_model(config: dict, seed: int = 0) -> Dict[str, torch.Tensor]:
    """bf16 checkpoint tensors of `config` (row scale ~ 1/sqrt(in), vectors off their neutral value)."""
    gen = torch.Generator().manual_seed(seed)

    def mat(out, inp, gain=1.0):
        return (torch.randn(out, inp, generator=gen) * (gain / math.sqrt(inp))).to(torch.bfloat16)

    def vec(n, center, spread=0.3):
        return (center + spread * torch.randn(n, generator=gen)).to(torch.bfloat16)

    def one(center):
        return vec(1, center)[0].clone()

    d = config["width"]
    w = {"embed": torch.randn(config["vocab"], d, generator=gen).to(torch.bfloat16),
         "head": mat(config["vocab"], d, 2.0), "final.norm": one(1.0)}
    for i, layer in enumerate(config["layers"]):
        m, p = layer["mixer"], f"l{i}."
        heads, vdim = m["heads"], m["vdim"]
        w[p + "norm1"] = one(1.0)
        p += "mix."
        w[p + "o"] = mat(d, heads * vdim)
        if layer["type"] == "latent_attention":
            w[p + "dq"], w[p + "dq.norm"] = mat(m["q_rank"], d), vec(m["q_rank"], 1.0)
            w[p + "uq"] = mat(heads * (m["dim"] + m["rot_dim"]), m["q_rank"], 2.0)
            if m.get("kv_from") is None:
                w[p + "dkv"] = mat(m["kv_rank"] + m["rot_dim"], d)
                w[p + "dkv.norm"] = vec(m["kv_rank"], 1.0)
            w[p + "uk"], w[p + "uv"] = mat(heads * m["dim"], m["kv_rank"], 2.0), mat(heads * vdim, m["kv_rank"])
            w[p + "sink"] = vec(heads, 0.5, 1.0)
            w[p + "g"] = mat(heads, d, 2.0)
        elif layer["type"] == "hgrn2":
            n = heads * m["dim"]
            w[p + "q"], w[p + "f"], w[p + "v"] = mat(n, d), mat(n, d, 2.0), mat(heads * vdim, d)
            w[p + "f.b"] = vec(n, 2.0, 1.5)
            w[p + "lower"] = torch.rand(n, generator=gen).mul(0.9).to(torch.bfloat16)
            w[p + "norm"] = vec(vdim, 1.0)
        else:
            inner, gn = heads * vdim, m["groups"] * m["state"]
            w[p + "in"] = mat(2 * inner + 2 * gn + heads, d)
            w[p + "conv"], w[p + "conv.b"] = mat(inner + 2 * gn, m["conv"], 1.5), vec(inner + 2 * gn, 0.0)
            w[p + "dt_bias"], w[p + "A_log"], w[p + "D"] = vec(heads, -1.0, 1.0), vec(heads, -0.5, 1.0), vec(heads, 1.0)
            w[p + "norm"] = vec(inner, 1.0)
        if layer.get("mlp") is not None:
            p = f"l{i}."
            ff = layer["mlp"]["ff"]
            w[p + "norm2"] = one(1.0)
            w[p + "mlp.up"], w[p + "mlp.up.b"] = mat(ff, d), vec(ff, 0.0)
            w[p + "mlp.down"], w[p + "mlp.down.b"] = mat(d, ff), vec(d, 0.0)
            w[p + "mlp.act"] = vec(2, 0.3, 0.5)
    return w


def config_dict(vocab=97, width=40, eps=1e-6, scale=1.7, mult=0.6, layers=()) -> dict:
    return {"architecture": "Soselix", "embedding": {"scale": scale}, "layers": [dict(l) for l in layers],
            "norm": {"eps": eps}, "residual_mult": mult, "vocab": vocab, "width": width}


def _ff(ff) -> Optional[dict]:
    return None if ff is None else {"ff": ff, "kind": "dense"}


def latent_layer(heads=6, dim=16, vdim=12, kv_rank=40, q_rank=24, rot_dim=8, base=500.0, scale=0.2, kv_from=None,
                 ff=56) -> dict:
    m = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "rot_dim": rot_dim,
         "rot": {"base": base, "dims": rot_dim}, "scale": scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mlp": _ff(ff), "mixer": m}


def hgrn_layer(heads=3, dim=12, vdim=20, ff=None) -> dict:
    return {"type": "hgrn2", "mlp": _ff(ff), "mixer": {"heads": heads, "dim": dim, "vdim": vdim}}


def mamba_layer(heads=4, vdim=12, state=20, groups=2, conv=4, norm_groups=3, ff=24) -> dict:
    return {"type": "mamba2", "mlp": _ff(ff),
            "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                      "norm_groups": norm_groups}}


def save_model(path, config: dict, weights: Dict[str, torch.Tensor]) -> None:
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(config, f)
    save_file({k: v.contiguous() for k, v in weights.items()}, os.path.join(path, "model.safetensors"))
