"""Native Tulezen decoder block: latent attention and routed experts, both
normed on their OUTPUT only:

    x <- x + norm1(mixer(x));   x <- x + norm2(experts(x))

with the residual x in 32-bit and norms scaled by (1 + weight).

What a token leaves in the cache is its latent c (kv_rank values); keys and
values are projections of c, so a block with ``kv_from`` owns no cache and reads
the latents of an earlier block, which must be served by the same server in the
same session (TulezenConfig.valid_cuts).

Two forward contracts:
  * ``forward_paged(x, batch, pool)``: rows of any number of sequences, latents
    in a PagedPool (server/paged_cache.py). The serving path: fused HIP kernels
    on the GPU (ops/latent.py), torch reference ops on the CPU.
  * ``forward(hidden, shared=...)``: whole sequences [B, S, D], differentiable,
    no cache; ``shared`` carries latents between the blocks of one chain.
"""

from __future__ import annotations

from typing import Dict, Optional

import torch
import torch.nn.functional as F
from torch import nn

from petals_amd.models.tulezen.config import TulezenConfig
from petals_amd.ops import reference


class TulezenBlock(nn.Module):
    paged = True
    _fast = None  # ops.latent.LatentMoEFastPath after optimize_for_inference()

    def __init__(self, config: TulezenConfig, layer_idx: int = 0):
        super().__init__()
        self.config = config
        self.layer_idx = layer_idx
        spec = config.spec(layer_idx)
        self.attention, self.moe, self.eps = spec.attention, spec.moe, config.layer_norm_eps
        self.source_layer = layer_idx if spec.attention.kv_from is None else spec.attention.kv_from
        d, a = config.hidden_size, spec.attention

        def param(*shape):
            return nn.Parameter(torch.zeros(*shape))

        self.norm1 = param(d)
        self.q = param(a.heads * a.dim, d)
        if a.kv_from is None:
            self.dkv = param(a.kv_rank, d)
            self.dkv_norm = param(a.kv_rank)
        self.uk = param(a.heads * a.dim, a.kv_rank)
        self.uv = param(a.heads * a.vdim, a.kv_rank)
        self.o = param(d, a.heads * a.vdim)
        if self.moe is not None:
            m = self.moe
            self.norm2 = param(d)
            self.router = param(m.experts, d)
            self.gate = param(m.experts, m.ff, d)
            self.up = param(m.experts, m.ff, d)
            self.down = param(m.experts, d, m.ff)

    # zero-centered norm weights start at 0, not 1 (server/from_pretrained.py)
    neutral_at_zero = frozenset({"norm1", "norm2"})

    def convert_state_dict(self, tensors: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
        """Checkpoint tensors of this block (prefix removed) -> parameters.
        Experts are stacked; a missing or misshapen tensor is an error."""
        names = {"norm1": "norm1", "q": "mix.q", "uk": "mix.uk", "uv": "mix.uv", "o": "mix.o"}
        if self.attention.kv_from is None:
            names.update({"dkv": "mix.dkv", "dkv_norm": "mix.dkv.norm"})
        if self.moe is not None:
            names.update({"norm2": "norm2", "router": "mlp.router"})
        out = {}
        try:
            for ours, theirs in names.items():
                out[ours] = tensors[theirs]
            if self.moe is not None:
                for kind in ("gate", "up", "down"):
                    out[kind] = torch.stack([tensors[f"mlp.e{e}.{kind}"] for e in range(self.moe.experts)])
        except KeyError as e:
            raise KeyError(f"block {self.layer_idx}: checkpoint has no tensor {e.args[0]!r}") from None
        for name, p in self.named_parameters():
            if tuple(out[name].shape) != tuple(p.shape):
                raise ValueError(
                    f"block {self.layer_idx}: {name} is {tuple(out[name].shape)}, config says {tuple(p.shape)}"
                )
        return out

    def optimize_for_inference(self, quant: str = "none") -> "TulezenBlock":
        """Repack the weights for the HIP kernels (frees the originals)."""
        from petals_amd.ops.latent import LatentMoEFastPath

        if quant != "none":
            raise ValueError(f"tulezen blocks are served in bfloat16 or float32, not quantized ({quant!r})")
        self._fast = LatentMoEFastPath(self)
        return self

    # ------------------------------------------------------------ cache spec

    def paged_cache_width(self) -> Optional[int]:
        """Padded latent size of the cache this block OWNS; None if it reads another's."""
        return self.config.cache_values_per_token(self.layer_idx) or None

    def weight(self, name: str) -> torch.Tensor:
        return getattr(self, name) if self._fast is None else self._fast.weight(name)

    # --------------------------------------------------------------- serving

    def forward_paged(self, x: torch.Tensor, batch, pool) -> torch.Tensor:
        """x [T, D] 32-bit residual of the batch's rows; returns the new one."""
        cache = pool.layer(self.source_layer)
        if self._fast is not None:
            return self._fast.forward_paged(x, batch, cache)
        if x.is_cuda:
            raise RuntimeError("a block on the GPU needs optimize_for_inference() before it serves")
        h = x.to(self.q.dtype)
        if self.attention.kv_from is None:
            c = reference.rms_norm((h @ self.dkv.T).float(), self.dkv_norm.float(), self.eps)
            reference.paged_write(cache, batch, c.to(cache.dtype))
        a = self.attention
        q = (h @ self.q.T).view(-1, a.heads, a.dim)
        y = reference.latent_attention_paged(
            q, cache, batch, self.uk, self.uv, scale=a.scale, window=a.window
        ).to(h.dtype)
        y = y.reshape(x.shape[0], a.heads * a.vdim) @ self.o.T
        x = x + reference.zero_centered_rms_norm(y, self.norm1, self.eps)
        return self._add_experts(x)

    # ----------------------------------------------------- stateless forward

    def forward(
        self,
        hidden_states: torch.Tensor,
        kv_cache=None,
        prefix_length: int = 0,
        ctx=None,
        shared: Optional[Dict[int, torch.Tensor]] = None,
    ) -> torch.Tensor:
        assert kv_cache is None and prefix_length == 0, "cached inference goes through forward_paged"
        a, eps = self.attention, self.eps
        b, s, d = hidden_states.shape
        x = hidden_states.float()
        h = x.to(self.weight("uk").dtype)
        if a.kv_from is None:
            c = reference.rms_norm((h @ self.weight("dkv").T).float(), self.weight("dkv_norm").float(), eps).to(h.dtype)
            if shared is not None:
                shared[self.layer_idx] = c
        elif shared is None or a.kv_from not in shared:
            raise ValueError(f"block {self.layer_idx} needs the latent of block {a.kv_from} from the same chain")
        else:
            c = shared[a.kv_from]
        q = (h @ self.weight("q").T).view(b, s, a.heads, a.dim)
        k = (c @ self.weight("uk").T).view(b, s, a.heads, a.dim)
        v = (c @ self.weight("uv").T).view(b, s, a.heads, a.vdim)
        mask = reference.sliding_window_mask(s, s, 0, a.window, x.device)
        y = reference.masked_attention(q, k, v, mask, a.scale).to(h.dtype)
        y = y.reshape(b, s, a.heads * a.vdim) @ self.weight("o").T
        x = x + reference.zero_centered_rms_norm(y, self.weight("norm1"), eps)
        return self._add_experts(x.reshape(b * s, d)).view(b, s, d)

    def _add_experts(self, x: torch.Tensor) -> torch.Tensor:
        """x [T, D]: x + norm2(experts(x)), torch ops."""
        if self.moe is None:
            return x
        m = self.moe
        weights, chosen = reference.softmax_topk(x, self.weight("router"), m.top)
        gate, up, down = self.weight("gate"), self.weight("up"), self.weight("down")
        h = x.to(gate.dtype)
        out = torch.zeros_like(x)
        for e in range(m.experts):
            rows, slots = torch.where(chosen == e)
            if rows.numel() == 0:
                continue
            he = h[rows]
            act = reference.clamped_swiglu(F.linear(he, gate[e]), F.linear(he, up[e]), m.limit).to(h.dtype)
            y = F.linear(act, down[e]).float() * weights[rows, slots, None]
            out = out.index_add(0, rows, y)
        return x + reference.zero_centered_rms_norm(out, self.weight("norm2"), self.eps)
