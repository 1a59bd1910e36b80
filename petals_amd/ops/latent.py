"""MI355X fast path of blocks with latent attention, routed experts and norms on
the sublayer outputs (models/tulezen).

Kernels: ops/csrc/latent_attn.hip, sublayer.hip, moe.hip, gemv.hip, in a library
of their own (ops/build.py "latent").

Everything per head is carried in LATENT space: W_uk is applied to the query and
W_uv to the attended latent, so attention reads the cached rows themselves and
all heads share them. Weights are padded once, at load, to the tile sizes of the
kernels (head sizes and latent to 32, width to 128, expert size to 64) with
zeros that contribute nothing; any size works, and none is assumed.

A batch takes one of two routes, whatever mix of requests it holds:
  few rows   split-K GEMVs, device-routed expert GEMVs; no library product and
             no host synchronisation, so the engine captures it in a hipGraph
  many rows  hipBLASLt products, expert-grouped MFMA GEMM
In float32 every product is a true 32-bit one.
"""

from __future__ import annotations

import torch

from petals_amd.ops.fused_decode import _EPI_PLAIN_F32

GATE_ALPHA = 1.702
_EPI_CLAMPED_SWIGLU_F32 = 5
_MOE_TILE = 32  # rows of a moe_gemm tile
_GEMV_ROWS = 8  # most rows of the dense GEMV
_MOE_GEMV_ROWS = 64  # most (token, slot) rows of the expert GEMV



def hip():
    """The compiled kernels; on a GPU there is nothing else to fall back to."""
    from petals_amd.ops import _hip

    return _hip.first_loaded("latent")


def _up(n: int, to: int) -> int:
    return -(-n // to) * to


def zero_centered_rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    rows = x.float().reshape(-1, x.shape[-1]).contiguous()
    out, _, _, _ = hip().sublayer_out(rows, None, weight.float().contiguous(), eps, None, rows.shape[1], False, None, 1)
    return out.view(x.shape)


class LatentMoEFastPath:
    quant = "none"

    def __init__(self, block):
        self.hip = hip()
        self.spec_a, self.spec_m, self.eps = block.attention, block.moe, block.eps
        a, m = self.spec_a, self.spec_m
        dtype, dev = block.q.dtype, block.q.device
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"latent attention is served in bfloat16 or float32, not {dtype}")
        self.dtype, self.f32 = dtype, dtype == torch.float32
        self.d = block.config.hidden_size
        self.dp = _up(self.d, 128)
        self.rank, self.rp = a.kv_rank, _up(a.kv_rank, 32)
        self.dim_p, self.vdim_p = _up(a.dim, 32), _up(a.vdim, 32)
        self.nq = a.heads * self.dim_p
        self.owns_latent = a.kv_from is None

        def zeros(*shape):
            return torch.zeros(*shape, dtype=dtype, device=dev)

        def f32(p):
            return p.detach().float().contiguous()

        # [in, out]: queries (heads padded), then the latent's rows
        n_in = self.nq + (_up(self.rank, 8) if self.owns_latent else 0)
        self.w_in = zeros(self.dp, n_in)
        q = block.q.detach().view(a.heads, a.dim, self.d)
        self.w_in[: self.d, : self.nq].view(self.d, a.heads, self.dim_p)[:, :, : a.dim] = q.permute(2, 0, 1)
        if self.owns_latent:
            self.w_in[: self.d, self.nq : self.nq + self.rank] = block.dkv.detach().t()
            self.latent_norm = f32(block.dkv_norm)
        # [H, RP, dim]: query into latent space;  [H, vdim, RP]: latent to value
        self.w_uk = zeros(a.heads, self.rp, self.dim_p)
        self.w_uk[:, : self.rank, : a.dim] = block.uk.detach().view(a.heads, a.dim, self.rank).transpose(1, 2)
        self.w_uv = zeros(a.heads, self.vdim_p, self.rp)
        self.w_uv[:, : a.vdim, : self.rank] = block.uv.detach().view(a.heads, a.vdim, self.rank)
        self.w_o = zeros(a.heads * self.vdim_p, self.dp)
        self.w_o.view(a.heads, self.vdim_p, self.dp)[:, : a.vdim, : self.d] = (
            block.o.detach().view(self.d, a.heads, a.vdim).permute(1, 2, 0)
        )
        self.norm1 = f32(block.norm1)
        self.max_gemv_rows = _GEMV_ROWS
        if m is not None:
            self.ffp = _up(m.ff, 64)
            self.w_router = zeros(m.experts, self.dp)
            self.w_router[:, : self.d] = block.router.detach()
            self.w_gu = zeros(m.experts, self.dp, 2 * self.ffp)
            self.w_gu[:, : self.d, : m.ff] = block.gate.detach().transpose(1, 2)
            self.w_gu[:, : self.d, self.ffp : self.ffp + m.ff] = block.up.detach().transpose(1, 2)
            self.w_down = zeros(m.experts, self.ffp, self.dp)
            self.w_down[:, : m.ff, : self.d] = block.down.detach().transpose(1, 2)
            self.norm2 = f32(block.norm2)
            self.max_gemv_rows = min(_GEMV_ROWS, _MOE_GEMV_ROWS // m.top)
        # batches that the engine may capture: only kernels of this library run
        self.max_graph_rows = 0 if self.f32 else self.max_gemv_rows
        self.graph_safe = self.max_graph_rows > 0
        self._no_ws = torch.empty(0, dtype=torch.float32, device=dev)
        empty = torch.empty(0, dtype=dtype, device=dev)
        for p in block.parameters():
            p.data = empty

    def weight(self, name: str) -> torch.Tensor:
        """A checkpoint-shaped view of a packed weight (stateless forward, backward)."""
        a, m, d = self.spec_a, self.spec_m, self.d
        if name == "q":
            return self.w_in[:d, : self.nq].view(d, a.heads, self.dim_p)[:, :, : a.dim].reshape(d, -1).t()
        if name == "dkv":
            return self.w_in[:d, self.nq : self.nq + self.rank].t()
        if name == "dkv_norm":
            return self.latent_norm
        if name == "uk":
            return self.w_uk[:, : self.rank, : a.dim].transpose(1, 2).reshape(a.heads * a.dim, self.rank)
        if name == "uv":
            return self.w_uv[:, : a.vdim, : self.rank].reshape(a.heads * a.vdim, self.rank)
        if name == "o":
            return self.w_o.view(a.heads, self.vdim_p, self.dp)[:, : a.vdim, :d].reshape(a.heads * a.vdim, d).t()
        if name in ("norm1", "norm2"):
            return getattr(self, name)
        if name == "router":
            return self.w_router[:, :d]
        if name == "gate":
            return self.w_gu[:, :d, : m.ff].transpose(1, 2)
        if name == "up":
            return self.w_gu[:, :d, self.ffp : self.ffp + m.ff].transpose(1, 2)
        if name == "down":
            return self.w_down[:, : m.ff, :d].transpose(1, 2)
        raise KeyError(name)

    # ---------------------------------------------------------------- forward

    def _dense(self, x: torch.Tensor, w: torch.Tensor, few: bool) -> torch.Tensor:
        """x [T, in] (32-bit if few rows or float32, else the weight dtype) @ w [in, out]."""
        if few:
            # 64 input rows a wave keeps the loads of a short gemv in flight
            splits = max(1, min(w.shape[0] // 64, 1024 // (-(-w.shape[1] // 512))))
            return self.hip.gemv_bf16(w, x, self._no_ws, None, _EPI_PLAIN_F32, splits)
        return x @ w

    def forward_paged(self, x: torch.Tensor, batch, cache: torch.Tensor) -> torch.Tensor:
        a, m, h = self.spec_a, self.spec_m, self.hip
        t = x.shape[0]
        few = not self.f32 and t <= self.max_gemv_rows
        dense_dtype = torch.float32 if few or self.f32 else self.dtype
        if self.dp != self.d:
            x = torch.nn.functional.pad(x, (0, self.dp - self.d))
        x = x.contiguous()

        # ---- latent attention
        y = self._dense(x.to(dense_dtype), self.w_in, few)
        if self.owns_latent:
            h.latent_write(y, self.nq, self.latent_norm, cache, batch.pos, batch.owner, batch.tables, self.eps)
        q = h.batched_linear(y[:, : self.nq].view(t, a.heads, self.dim_p), self.w_uk, self.f32)
        run = batch.run_tokens(a.heads)
        max_keys = min(batch.max_end, a.window) if a.window > 0 else batch.max_end
        lat = h.latent_attention(
            q, cache, batch.pos, batch.owner, batch.tables, batch.tiles(run), run, max_keys, a.window, a.scale
        )
        o = h.batched_linear(lat, self.w_uv, dense_dtype == torch.float32).view(t, a.heads * self.vdim_p)
        y = self._dense(o, self.w_o, few)
        want_bf16 = m is not None and not few and not self.f32
        router = self.w_router if m is not None else None
        x, xb, sel, scores = h.sublayer_out(
            y, None, self.norm1, self.eps, x, self.dp, want_bf16, router, m.top if m is not None else 1
        )

        # ---- routed experts
        if m is not None:
            pairs = sel.view(-1)
            if self.f32:
                act = h.clamped_swiglu(h.moe_linear_f32(self.w_gu, x, pairs, m.top), m.limit, GATE_ALPHA)
                y = h.moe_linear_f32(self.w_down, act, pairs, 1)
            elif few:
                act = h.gemv_bf16_moe(
                    self.w_gu, x, pairs, m.top, self._no_ws, _EPI_CLAMPED_SWIGLU_F32, 0, m.limit, GATE_ALPHA
                )
                y = h.gemv_bf16_moe(self.w_down, act, pairs, 1, self._no_ws, _EPI_PLAIN_F32)
            else:
                order, tile_expert = h.moe_group(pairs, m.experts, _MOE_TILE)
                gu = h.moe_gemm(self.w_gu, None, None, xb, order, tile_expert, m.top, t * m.top)
                act = h.clamped_swiglu(gu, m.limit, GATE_ALPHA)
                y = h.moe_gemm(self.w_down, None, None, act, order, tile_expert, 1, t * m.top)
            x, _, _, _ = h.sublayer_out(y, scores, self.norm2, self.eps, x, self.dp, False, None, 1)
        return x[:, : self.d] if self.dp != self.d else x
