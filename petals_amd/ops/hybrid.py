"""MI355X fast path of pre-norm blocks with windowed attention or a gated delta
rule and a dense feed-forward (models/lefulorn).

Kernels: ops/csrc/paged_attn.hip, delta.hip, prenorm.hip, gemv.hip, in a library
of their own (ops/build.py "hybrid").

Everything that reads the normed input is one product: queries, keys, values and
gate of attention; queries, keys, values, beta and the inner low-rank projections
of the delta rule. Weights are padded once, at load, to the tile sizes of the
kernels with zeros that contribute nothing; any size works, and none is assumed.

A batch takes one of two routes, whatever mix of requests it holds:
  few rows   split-K GEMVs with 32-bit activations; no library product and no host
             synchronisation, so the engine captures single-token batches in a
             hipGraph
  many rows  hipBLASLt products
In float32 every product is a true 32-bit one. The delta rule has a kernel for
batches of single tokens and a chunked one for all others.
"""

from __future__ import annotations

import torch

from petals_amd.models.lefulorn.config import KEY_PAD, VALUE_PAD
from petals_amd.ops import reference
from petals_amd.ops.fused_decode import _EPI_PLAIN_F32

_EPI_RELU2_F32 = 6
_EPI_RAW = -1  # the split-K partial sums
_GEMV_ROWS = 8  # most rows of the GEMV
_CHUNK = 16  # tokens of a chunk of the delta rule


def hip():
    """The compiled kernels; on a GPU there is nothing else to fall back to."""
    from petals_amd.ops import _hip

    return _hip.first_loaded("hybrid")


def _up(n: int, to: int) -> int:
    return -(-n // to) * to


def rms_norm_f32(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    d = x.shape[-1]
    rows = x.float().reshape(-1, d).contiguous()
    return hip().residual_norm(rows, None, None, weight.float().contiguous(), d, eps, True)[:, :d].reshape(x.shape)


class HybridFastPath:
    quant = "none"

    def __init__(self, block):
        self.hip = hip()
        self.spec, self.mlp, self.eps, self.mix = block.mixer, block.mlp, block.eps, block.mix
        dtype, dev = block.q.dtype, block.q.device
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"these blocks are served in bfloat16 or float32, not {dtype}")
        self.dtype, self.f32, self.device = dtype, dtype == torch.float32, dev
        self.d = block.config.hidden_size
        self.dp = _up(self.d, 8)
        self.carried = block.config.carried_values
        self._views = {}  # checkpoint-shaped views of packed weights
        self.norm1 = self._f32(block, "norm1")
        if block.delta:
            self._pack_delta(block)
        else:
            self._pack_attention(block)
        if self.mlp is not None:
            self.norm2 = self._f32(block, "norm2")
            ffp = _up(self.mlp.ff, 8)
            self.w_up, self.w_down = self._zeros(self.dp, ffp), self._zeros(ffp, self.dp)
            self._place(block, "up", self.w_up[: self.d, : self.mlp.ff].t())
            self._place(block, "down", self.w_down[: self.mlp.ff, : self.d].t())
            self.b_up = torch.zeros(ffp, device=dev)
            self._place(block, "up_bias", self.b_up[: self.mlp.ff])
            self.b_down = self._f32(block, "down_bias")
            self.b_up_gemv = self.b_up.to(torch.bfloat16)
        self.max_gemv_rows = _GEMV_ROWS
        # batches that the engine may capture: only kernels of this library run
        self.max_graph_rows = 0 if self.f32 or not self.captures else self.max_gemv_rows
        self.graph_safe = self.max_graph_rows > 0
        self._no_ws = torch.empty(0, dtype=torch.float32, device=dev)
        empty = torch.empty(0, dtype=dtype, device=dev)
        for p in block.parameters():
            p.data = empty

    # ---------------------------------------------------------------- weights

    def _zeros(self, *shape):
        return torch.zeros(*shape, dtype=self.dtype, device=self.device)

    def _f32(self, block, name):
        t = getattr(block, name).detach().float().contiguous()
        self._views[name] = t
        return t

    def _place(self, block, name, view):
        """Copy a parameter into its place in a packed weight."""
        view.copy_(getattr(block, name).detach().view(view.shape))
        self._views[name] = view

    def weight(self, name: str) -> torch.Tensor:
        """A checkpoint-shaped weight (stateless forward, backward)."""
        view = self._views[name]
        if view.dim() == 3:  # padded heads
            view = view.reshape(-1, view.shape[-1]) if name != "o" else view.reshape(view.shape[0], -1)
        return view

    def _columns(self, block, parts):
        """w_in [dp, n]: the named weights [out, d] side by side; parts: (name, heads,
        size, padded size). Returns each part's first column."""
        starts, n = [], 0
        for _, heads, _, padded in parts:
            starts.append(n)
            n += _up(heads * padded, 8)
        self.w_in = self._zeros(self.dp, n)
        for at, (name, heads, size, padded) in zip(starts, parts):
            heads_view = self.w_in[: self.d, at : at + heads * padded].unflatten(1, (heads, padded))[:, :, :size]
            self._place(block, name, heads_view.permute(1, 2, 0))
        return starts

    def _pack_attention(self, block):
        a = self.spec
        self.dk, self.dv = _up(a.dim, KEY_PAD), _up(a.vdim, VALUE_PAD)
        _, at_k, at_v, self.at_gate = self._columns(block, [
            ("q", a.heads, a.dim, self.dk), ("k", a.kv_heads, a.dim, self.dk), ("v", a.kv_heads, a.vdim, self.dv),
            ("g", a.heads, a.vdim, self.dv),
        ])
        self.b_in = torch.zeros(self.at_gate, device=self.device)
        for name, at, heads, size, padded in (
            ("q_bias", 0, a.heads, a.dim, self.dk), ("k_bias", at_k, a.kv_heads, a.dim, self.dk),
            ("v_bias", at_v, a.kv_heads, a.vdim, self.dv),
        ):
            view = self.b_in[at : at + heads * padded].view(heads, padded)[:, :size]
            self._place(block, name, view)
            self._views[name] = view.reshape(-1)
        self.w_o = self._zeros(a.heads * self.dv, self.dp)
        self._place(block, "o", self.w_o.view(a.heads, self.dv, self.dp)[:, : a.vdim, : self.d].permute(2, 0, 1))
        self.sink = self._f32(block, "sink")
        self.slopes = reference.distance_slopes(a.heads, self.device)
        self.lam = self._f32(block, "vmix") if self.mix == "mix" else None
        self.captures = self.dk <= 256 and self.dv <= 256

    def _pack_delta(self, block):
        m = self.spec
        a_rank, g_rank = block.a1.shape[0], block.g1.shape[0]
        *self.cols, self.at_a1, self.at_g1 = self._columns(block, [
            ("q", m.kv_heads, m.dim, m.dim), ("k", m.kv_heads, m.dim, m.dim), ("v", m.heads, m.vdim, m.vdim),
            ("b", m.heads, 1, 1), ("a1", 1, a_rank, _up(a_rank, 8)), ("g1", 1, g_rank, _up(g_rank, 8)),
        ])
        self.w_a2 = self._zeros(m.heads * m.dim, _up(a_rank, 8))
        self.w_g2 = self._zeros(m.heads * m.vdim, _up(g_rank, 8))
        self._place(block, "a2", self.w_a2[:, :a_rank])
        self._place(block, "g2", self.w_g2[:, :g_rank])
        # [taps, channels]
        conv_w = torch.cat([getattr(block, f"{n}_conv").detach().float() for n in ("q", "k", "v")])
        self.conv_w = conv_w.t().contiguous()
        rows = [getattr(block, f"{n}_conv").shape[0] for n in ("q", "k", "v")]
        self._views.update(zip(("q_conv", "k_conv", "v_conv"), self.conv_w.t().split(rows)))
        self.a_exp = self._f32(block, "A_log").exp()
        self.dt_bias, self.o_norm = self._f32(block, "dt_bias"), self._f32(block, "o_norm")
        self.wide = _up(m.heads * m.vdim, 8)
        self.w_o = self._zeros(self.wide, self.dp)
        self._place(block, "o", self.w_o[: m.heads * m.vdim, : self.d].t())
        self.captures = self.hip.delta_decodes(m.dim, m.vdim)

    # ---------------------------------------------------------------- forward

    def _splits(self, w: torch.Tensor) -> int:
        # 64 input rows a wave keeps the loads of a short gemv in flight
        return max(1, min(w.shape[0] // 64, 1024 // (-(-w.shape[1] // 512))))

    def _dense(self, x, w, few: bool, epilogue: int = _EPI_PLAIN_F32, bias=None):
        """x [T, in] (32-bit if few rows or float32, else the weight dtype) @ w [in, out]."""
        if few:
            return self.hip.gemv_bf16(w, x, self._no_ws, None, epilogue, self._splits(w), bias)
        return x @ w

    def _add(self, x, y, w, few: bool, bias=None):
        """x += y @ w (+ bias), for the last product before x is read again."""
        if few:
            self.hip.residual_sum(self._dense(y, w, True, _EPI_RAW), bias, x, self.d)
        else:
            self.hip.residual_norm(x, y @ w, bias, None, self.d, self.eps, True)

    def forward_paged(self, x: torch.Tensor, batch, cache=None, state=None) -> torch.Tensor:
        """x [T, stream width] 32-bit, updated in place."""
        h = self.hip
        few = not self.f32 and x.shape[0] <= self.max_gemv_rows
        wide = few or self.f32  # 32-bit activations
        y = self._dense(h.residual_norm(x, None, None, self.norm1, self.d, self.eps, wide), self.w_in, few)
        y = self._attention(x, y, batch, cache, wide) if state is None else self._delta(y, batch, state, wide)
        if self.mlp is None:
            self._add(x, y, self.w_o, few)
            return x
        if few:
            self._add(x, y, self.w_o, few)
            n = h.residual_norm(x, None, None, self.norm2, self.d, self.eps, wide)
            act = self._dense(n, self.w_up, few, _EPI_RELU2_F32, self.b_up_gemv)
        else:
            n = h.residual_norm(x, y @ self.w_o, None, self.norm2, self.d, self.eps, wide)
            act = h.bias_relu2(n @ self.w_up, self.b_up)
        self._add(x, act, self.w_down, few, self.b_down)
        return x

    def _attention(self, x, y, batch, cache, wide):
        a, h = self.spec, self.hip
        first = x[:, self.d :] if self.mix else None
        q = h.attn_prepare(
            y, self.b_in, cache, batch.pos, batch.owner, batch.tables, a.heads, a.kv_heads, self.dk, self.dv,
            a.temp_coef, a.temp_every, first, self.lam, a.vdim,
        )
        group = a.heads // a.kv_heads
        run = batch.run_tokens(group)
        max_keys = min(batch.max_end, a.window) if a.window > 0 else batch.max_end
        return h.paged_attention(
            q, cache, batch.pos, batch.owner, batch.tables, batch.tiles(run), run, max_keys, a.kv_heads, self.dv,
            a.window, a.scale, self.slopes, self.sink, y[:, self.at_gate : self.at_gate + a.heads * self.dv], wide,
        )

    def _delta(self, y, batch, state, wide):
        m, h = self.spec, self.hip
        delta, conv = state["delta"], state["conv"]
        sizes = (m.heads, m.kv_heads, m.dim, m.vdim, self.cols)
        if batch.decode_only and self.captures:
            return h.delta_decode(
                y, self.conv_w, self.w_a2, self.w_g2, self.at_a1, self.at_g1, self.a_exp, self.dt_bias, self.o_norm,
                batch.pos, batch.slot, delta, conv, *sizes, self.wide, self.eps,
            )
        a, gate = (
            self._outer(y[:, at : at + w.shape[1]], w) for at, w in ((self.at_a1, self.w_a2), (self.at_g1, self.w_g2))
        )
        o = h.delta_prefill(
            y, a, self.conv_w, self.a_exp, self.dt_bias, batch.tiles(_CHUNK), batch.chunk_bounds(_CHUNK), batch.pos,
            batch.owner, batch.slot, delta, conv, *sizes,
        )
        return h.delta_norm(o, gate, self.o_norm, m.heads, self.wide, wide, self.eps)

    def _outer(self, x, w):
        """x [T, rank] @ w [n, rank].T with a 32-bit result."""
        if self.f32:
            return x @ w.t()
        return self.hip.batched_linear(x.unsqueeze(1), w.unsqueeze(0), True).squeeze(1)
