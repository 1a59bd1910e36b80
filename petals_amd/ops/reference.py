"""Pure-PyTorch reference implementations of every op in the HIP kernel suite.

These are (a) the CPU execution path, and (b) the numerics baseline the HIP
kernels are exact-match tested against (fp32). Keep them obviously correct and
boring; performance lives in `petals_amd/ops/csrc/*.hip`.
"""

from __future__ import annotations

import math
from typing import Optional, Tuple

import torch
import torch.nn.functional as F


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float = 1e-5) -> torch.Tensor:
    dtype = x.dtype
    x32 = x.to(torch.float32)
    variance = x32.pow(2).mean(-1, keepdim=True)
    x32 = x32 * torch.rsqrt(variance + eps)
    return (x32 * weight.to(torch.float32)).to(dtype)


def build_rope_cache(
    head_dim: int,
    max_len: int,
    theta: float = 10000.0,
    device=None,
    dtype=torch.float32,
    rope_scaling: Optional[dict] = None,
) -> Tuple[torch.Tensor, torch.Tensor]:
    """cos/sin tables of shape [max_len, head_dim] (half-dim duplicated, HF
    rotate-half convention). Supports llama3 and linear rope scaling."""
    inv_freq = 1.0 / (theta ** (torch.arange(0, head_dim, 2, dtype=torch.float32) / head_dim))
    if rope_scaling:
        rtype = rope_scaling.get("rope_type", rope_scaling.get("type", ""))
        if rtype == "linear":
            inv_freq = inv_freq / float(rope_scaling["factor"])
        elif rtype == "llama3":
            factor = float(rope_scaling["factor"])
            lo = float(rope_scaling.get("low_freq_factor", 1.0))
            hi = float(rope_scaling.get("high_freq_factor", 4.0))
            orig = float(rope_scaling.get("original_max_position_embeddings", 8192))
            wavelen = 2 * math.pi / inv_freq
            lo_wl, hi_wl = orig / lo, orig / hi
            scaled = torch.where(wavelen > lo_wl, inv_freq / factor, inv_freq)
            smooth = (orig / wavelen - lo) / (hi - lo)
            smoothed = (1 - smooth) / factor * inv_freq + smooth * inv_freq
            mid = (wavelen <= lo_wl) & (wavelen >= hi_wl)
            inv_freq = torch.where(mid, smoothed, scaled)
    t = torch.arange(max_len, dtype=torch.float32)
    freqs = torch.outer(t, inv_freq)  # [max_len, head_dim/2]
    emb = torch.cat([freqs, freqs], dim=-1)
    cos, sin = emb.cos().to(dtype), emb.sin().to(dtype)
    if device is not None:
        cos, sin = cos.to(device), sin.to(device)
    return cos, sin


def _rotate_half(x: torch.Tensor) -> torch.Tensor:
    half = x.shape[-1] // 2
    return torch.cat([-x[..., half:], x[..., :half]], dim=-1)


def apply_rope(
    q: torch.Tensor, k: torch.Tensor, cos: torch.Tensor, sin: torch.Tensor, position_ids: torch.Tensor
) -> Tuple[torch.Tensor, torch.Tensor]:
    """q,k: [batch, heads, len, head_dim]; position_ids: [batch, len] or [len]."""
    if position_ids.dim() == 1:
        position_ids = position_ids.unsqueeze(0)
    cos_g = cos[position_ids].unsqueeze(1).to(q.dtype)  # [b, 1, len, hd]
    sin_g = sin[position_ids].unsqueeze(1).to(q.dtype)
    q_out = q * cos_g + _rotate_half(q) * sin_g
    k_out = k * cos_g + _rotate_half(k) * sin_g
    return q_out, k_out


def repeat_kv(x: torch.Tensor, n_rep: int) -> torch.Tensor:
    """[b, kv_heads, len, hd] -> [b, kv_heads*n_rep, len, hd]."""
    if n_rep == 1:
        return x
    b, kvh, slen, hd = x.shape
    return x[:, :, None].expand(b, kvh, n_rep, slen, hd).reshape(b, kvh * n_rep, slen, hd)


def attention(
    q: torch.Tensor,
    k: torch.Tensor,
    v: torch.Tensor,
    *,
    causal: bool,
    kv_offset: int = 0,
    attn_bias: Optional[torch.Tensor] = None,
    scale: Optional[float] = None,
) -> torch.Tensor:
    """Reference attention with fp32 softmax.

    q: [b, n_heads, q_len, hd]; k/v: [b, n_kv_heads, kv_len, hd].
    `causal` masks position (i + kv_offset) < j for query i, key j.
    `kv_offset` is the absolute position of q[0] within the kv sequence
    (kv_len = kv_offset + q_len when attending over a cache).
    `attn_bias`: optional additive bias [b or 1, n_heads, q_len, kv_len] (ALiBi).
    """
    b, n_heads, q_len, hd = q.shape
    n_kv = k.shape[1]
    if n_kv != n_heads:
        k = repeat_kv(k, n_heads // n_kv)
        v = repeat_kv(v, n_heads // n_kv)
    if scale is None:
        scale = 1.0 / math.sqrt(hd)
    scores = torch.matmul(q.to(torch.float32), k.to(torch.float32).transpose(-1, -2)) * scale
    if attn_bias is not None:
        scores = scores + attn_bias.to(torch.float32)
    if causal and q_len > 1:
        kv_len = k.shape[2]
        q_pos = torch.arange(q_len, device=q.device)[:, None] + kv_offset
        k_pos = torch.arange(kv_len, device=q.device)[None, :]
        mask = k_pos > q_pos
        scores = scores.masked_fill(mask, float("-inf"))
    probs = torch.softmax(scores, dim=-1)
    out = torch.matmul(probs.to(v.dtype), v)
    return out


def swiglu(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
    return F.silu(gate) * up


def gelu(x: torch.Tensor) -> torch.Tensor:
    return F.gelu(x, approximate="tanh")


def build_alibi_slopes(n_heads: int) -> torch.Tensor:
    """ALiBi per-head slopes (same closed form as the ALiBi paper)."""

    def pow2_slopes(n):
        start = 2.0 ** (-(2.0 ** -(math.log2(n) - 3)))
        return [start * (start**i) for i in range(n)]

    if math.log2(n_heads).is_integer():
        slopes = pow2_slopes(n_heads)
    else:
        closest = 2 ** math.floor(math.log2(n_heads))
        slopes = pow2_slopes(closest)
        extra = pow2_slopes(2 * closest)
        slopes += extra[0::2][: n_heads - closest]
    return torch.tensor(slopes, dtype=torch.float32)


def build_alibi_bias(
    n_heads: int, q_len: int, kv_len: int, device=None, dtype=torch.float32
) -> torch.Tensor:
    """[1, n_heads, q_len, kv_len] additive bias: slope * (j - i_abs) for j <= i."""
    slopes = build_alibi_slopes(n_heads).to(device)
    k_pos = torch.arange(kv_len, device=device, dtype=torch.float32)
    # bloom-style: bias depends only on key position distance from the last axis
    bias = slopes[:, None, None] * k_pos[None, None, :]  # [heads, 1, kv_len]
    return bias.unsqueeze(0).to(dtype).expand(1, n_heads, q_len, kv_len)


# ------------------------------------------- latent attention, routed experts


def zero_centered_rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) * (1 + weight), 32-bit in and out."""
    x = x.float()
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps) * (1.0 + weight.float())


def clamped_swiglu(gate: torch.Tensor, up: torch.Tensor, limit: float, alpha: float = 1.702) -> torch.Tensor:
    """g * sigmoid(alpha g) * (u + 1) with g = min(gate, limit), |u| <= limit."""
    g = gate.float().clamp(max=limit)
    u = up.float().clamp(min=-limit, max=limit)
    return g * torch.sigmoid(alpha * g) * (u + 1.0)


def softmax_topk(x: torch.Tensor, w_router: torch.Tensor, top: int):
    """32-bit router: (scores [T, top], experts [T, top]); the scores are the
    softmax over ALL experts, not renormalized over the chosen ones."""
    return torch.topk(torch.softmax(x.float() @ w_router.float().T, dim=-1), top, dim=-1)


def sliding_window_mask(q_len: int, kv_len: int, kv_offset: int, window: int, device=None) -> torch.Tensor:
    """[q_len, kv_len] visibility: query i stands at kv_offset + i among the keys
    and sees itself and the window - 1 keys before it (window 0: all before)."""
    gap = (torch.arange(q_len, device=device) + kv_offset)[:, None] - torch.arange(kv_len, device=device)[None, :]
    return (gap >= 0) & (gap < window) if window > 0 else gap >= 0


def masked_attention(q, k, v, mask, scale: float) -> torch.Tensor:
    """q [..., Sq, H, d], k/v [..., Sk, H, d]; 32-bit scores, weights and output."""
    q, k, v = (t.transpose(-3, -2).float() for t in (q, k, v))
    scores = (q @ k.transpose(-1, -2)) * scale
    p = torch.softmax(scores.masked_fill(~mask, float("-inf")), dim=-1)
    return (p @ v).transpose(-3, -2)


def paged_write(cache: torch.Tensor, batch, rows: torch.Tensor) -> None:
    """Store one row per token of the batch in the paged cache [pages, page, width]."""
    page = cache.shape[1]
    for s, (lo, hi) in enumerate(batch.row_ranges()):
        pos = torch.arange(batch.starts[s], batch.starts[s] + hi - lo)
        pages = torch.as_tensor(batch.pages[s])[pos // page]
        cache[pages, pos % page, : rows.shape[1]] = rows[lo:hi].to(cache.dtype)


def latent_attention_paged(q, cache, batch, w_uk, w_uv, *, scale: float, window: int) -> torch.Tensor:
    """q [T, H, dim] of the batch's rows against the latents in the paged cache;
    returns [T, H, vdim], 32-bit."""
    t, heads, dim = q.shape
    rank, page = w_uk.shape[1], cache.shape[1]
    out = torch.empty(t, heads, w_uv.shape[0] // heads, dtype=torch.float32)
    for s, (lo, hi) in enumerate(batch.row_ranges()):
        start, n = batch.starts[s], hi - lo
        first = max(0, start - window + 1) if window > 0 else 0
        pos = torch.arange(first, start + n)
        c = cache[torch.as_tensor(batch.pages[s])[pos // page], pos % page, :rank].to(w_uk.dtype)
        k = (c @ w_uk.T).view(-1, heads, dim)
        v = (c @ w_uv.T).view(c.shape[0], heads, -1)
        mask = sliding_window_mask(n, len(pos), start - first, window)
        out[lo:hi] = masked_attention(q[lo:hi], k, v, mask, scale)
    return out


# --------------------------------- gated delta rule, attention with a sink


def short_conv(x: torch.Tensor, weight: torch.Tensor) -> torch.Tensor:
    """Causal convolution per channel: x [B, taps - 1 + S, C] with the inputs before
    the first output ahead, weight [C, taps] (last column: the current token)."""
    taps = weight.shape[1]
    s = x.shape[1] - taps + 1
    return sum(x[:, j : j + s] * weight[:, j] for j in range(taps))


def unit_vectors(x: torch.Tensor, eps: float = 1e-6) -> torch.Tensor:
    return x * torch.rsqrt(x.pow(2).sum(-1, keepdim=True) + eps)


def gated_delta_rule(q, k, v, g, beta, state=None):
    """q, k, g [B, S, H, dim], v [B, S, H, vdim], beta [B, S, H]; 32-bit. Per token
    S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q.
    Returns (o [B, S, H, vdim], last state [B, H, dim, vdim])."""
    b, s, h, dim = q.shape
    if state is None:
        state = torch.zeros(b, h, dim, v.shape[-1], device=q.device)
    out = []
    for t in range(s):
        state = g[:, t, :, :, None] * state
        u = beta[:, t, :, None] * (v[:, t] - torch.einsum("bhk,bhkv->bhv", k[:, t], state))
        state = state + k[:, t, :, :, None] * u[:, :, None, :]
        out.append(torch.einsum("bhk,bhkv->bhv", q[:, t], state))
    return torch.stack(out, dim=1), state


def distance_slopes(heads: int, device=None) -> torch.Tensor:
    """2^(-8 (h + 1) / heads), for any number of heads."""
    return torch.exp2(-8.0 * torch.arange(1, heads + 1, device=device).float() / heads)


def query_temperature(pos: torch.Tensor, coef: float, every: int) -> torch.Tensor:
    """1 + coef * ln(floor((p + 1) / every) + 1), 32-bit."""
    return 1.0 + coef * torch.log1p(((pos + 1) // every).float())


def biased_sink_attention(
    q, k, v, q_pos, k_pos, *, scale, window, sink, slopes=None, temperature=None
) -> torch.Tensor:
    """q [..., Sq, H, d], k/v [..., Sk, G, d]; a distance bias slope * (i - j) is taken
    off the scores, and the softmax's denominator holds exp(sink) per head. 32-bit."""
    group = q.shape[-2] // k.shape[-2]
    k, v = (t.float().repeat_interleave(group, dim=-2).transpose(-3, -2) for t in (k, v))
    q = (q.float() if temperature is None else q.float() * temperature[:, None, None]).transpose(-3, -2)
    gap = (q_pos[:, None] - k_pos[None, :]).float()
    score = (q @ k.transpose(-1, -2).contiguous()) * scale
    if slopes is not None:
        score = score - slopes[:, None, None] * gap
    seen = (gap >= 0) & (gap < window) if window > 0 else gap >= 0
    score = score.masked_fill(~seen, float("-inf"))
    sink = sink.float()[:, None, None].expand(*score.shape[:-1], 1)
    p = torch.softmax(torch.cat([score, sink], dim=-1), dim=-1)[..., :-1]
    return (p @ v).transpose(-3, -2)


# ------------------- rotated halves, gated linear attention, group norm, xIELU


def rotary_frequencies(dims: int, base: float, yarn=None, device=None):
    """(radians per position of each of dims/2 pairs, 64-bit; factor of cos and sin).
    yarn: an object with factor, original, fast and slow, or None."""
    i = torch.arange(dims // 2, device=device, dtype=torch.float64)
    freqs = base ** (-2.0 * i / max(dims, 1))
    if yarn is None or dims == 0:
        return freqs, 1.0

    def pair(turns):  # (2 x) the pair that turns this often over the original positions
        return dims * math.log(yarn.original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo, hi = max(math.floor(pair(yarn.fast)), 0), min(math.ceil(pair(yarn.slow)), dims - 1)
    ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
    return freqs / yarn.factor * ramp + freqs * (1.0 - ramp), 0.1 * math.log(yarn.factor) + 1.0


def rotate_pairs(x: torch.Tensor, pos: torch.Tensor, freqs: torch.Tensor, factor: float = 1.0) -> torch.Tensor:
    """x [..., n] at positions pos (broadcast over x's leading axes): pair (i, i + len(freqs))
    turns by pos * freqs[i] and grows by `factor`; the values behind the pairs pass."""
    half = len(freqs)
    if half == 0:
        return x
    angle = pos[..., None].double() * freqs
    cos, sin = (angle.cos() * factor).float(), (angle.sin() * factor).float()
    u, v, rest = x.split([half, half, x.shape[-1] - 2 * half], dim=-1)
    return torch.cat([u * cos - v * sin, v * cos + u * sin, rest], dim=-1)


def rotate_halves(x: torch.Tensor, pos: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """x [..., n] at positions pos (broadcast over x's leading axes): the pair
    (i, i + dims/2) of the first `dims` values turns by pos * base^(-2i/dims)."""
    return rotate_pairs(x, pos, rotary_frequencies(dims, base, device=x.device)[0])


def forget_gate(z: torch.Tensor, lower: torch.Tensor):
    """f = lower + (1 - lower) sigmoid(z); returns (1 - f, f), the first without cancellation."""
    return (1.0 - lower) * torch.sigmoid(-z), lower + (1.0 - lower) * torch.sigmoid(z)


def gated_linear_attention(q, k, v, g, state=None):
    """q, k [B, S, H, dim], v [B, S, H, vdim], g [B, S, H, dim or 1]; 32-bit. Per token
    S <- g S + k v^T;  o = S^T q. Returns (o [B, S, H, vdim], last state [B, H, dim, vdim])."""
    if state is None:
        state = torch.zeros(q.shape[0], q.shape[2], q.shape[3], v.shape[3], device=q.device)
    out = []
    for t in range(q.shape[1]):
        state = g[:, t, :, :, None] * state + k[:, t, :, :, None] * v[:, t, :, None, :]
        out.append(torch.einsum("bhk,bhkv->bhv", q[:, t], state))
    return torch.stack(out, dim=1), state


def group_rms_norm(x: torch.Tensor, weight: torch.Tensor, groups: int, eps: float) -> torch.Tensor:
    """RMS norm of each of `groups` equal parts of the last axis, one weight per value."""
    parts = x.unflatten(-1, (groups, -1))
    return (parts * torch.rsqrt(parts.pow(2).mean(-1, keepdim=True) + eps)).flatten(-2) * weight


def xielu(z: torch.Tensor, p: torch.Tensor, q: torch.Tensor) -> torch.Tensor:
    """z > 0: softplus(p) z^2 + z/2;  z <= 0: (1/2 + softplus(q)) (exp(z) - 1 - z) + z/2."""
    low = z.clamp(max=0.0)
    negative = (0.5 + F.softplus(q)) * (torch.expm1(low) - low)
    return torch.where(z > 0, F.softplus(p) * z * z, negative) + 0.5 * z


# ---------------- capped, differential and sigmoid attention, PolyNorm


def visible(q_pos: torch.Tensor, k_pos: torch.Tensor, chunk: int = 0) -> torch.Tensor:
    """[Sq, Sk]: keys at or before the query, in its own run of `chunk` positions (0: all of them)."""
    seen = k_pos[None, :] <= q_pos[:, None]
    if chunk > 0:
        seen = seen & (k_pos[None, :] // chunk == q_pos[:, None] // chunk)
    return seen


def scored_attention(q, k, v, seen, *, scale, softcap=0.0, sigmoid_bias=None) -> torch.Tensor:
    """q [..., Sq, H, d], k/v [..., Sk, G, d]; 32-bit. Scores are capped by a tanh if `softcap` is
    given; weights are a softmax, or sigmoids of scores plus a bias per head."""
    group = q.shape[-2] // k.shape[-2]
    q = q.float().transpose(-3, -2)
    k, v = (t.float().repeat_interleave(group, dim=-2).transpose(-3, -2) for t in (k, v))
    score = (q @ k.transpose(-1, -2).contiguous()) * scale
    if softcap > 0:
        score = softcap * torch.tanh(score / softcap)
    if sigmoid_bias is not None:
        p = torch.sigmoid(score + sigmoid_bias.float()[:, None, None]).masked_fill(~seen, 0.0)
    else:
        p = torch.softmax(score.masked_fill(~seen, float("-inf")), dim=-1)
    return (p @ v).transpose(-3, -2)


def differential_share(lq1, lk1, lq2, lk2, diff: float) -> torch.Tensor:
    """exp(lq1 . lk1) - exp(lq2 . lk2) + diff: how much of the second map is taken off the first."""
    first, second = ((a.float() * b.float()).sum().exp() for a, b in ((lq1, lk1), (lq2, lk2)))
    return first - second + diff


def poly_norm(z: torch.Tensor, act: torch.Tensor, eps: float) -> torch.Tensor:
    """a N(z) + b N(z^2) + c N(z^3) + e, act = (a, b, c, e); N divides a row by its root mean square."""
    one = z.new_ones(())
    a, b, c, e = act
    return a * rms_norm(z, one, eps) + b * rms_norm(z * z, one, eps) + c * rms_norm(z * z * z, one, eps) + e
