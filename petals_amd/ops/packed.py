"""What the fast paths of pre-norm blocks with a dense feed-forward have in common
(ops/hybrid.py, ops/recurrent.py, ops/scores.py): weights packed once at load, and the two routes
of a batch, whatever mix of requests it holds:

  few rows   split-K GEMVs with 32-bit activations; no library product and no host
             synchronisation, so the engine captures single-token batches in a
             hipGraph
  many rows  hipBLASLt products

In float32 every product is a true 32-bit one. Weights are padded with zeros that
contribute nothing to the tile sizes of the kernels; any size works, and none is
assumed.
"""

from __future__ import annotations

import torch

from petals_amd.ops.fused_decode import _EPI_PLAIN_F32

_EPI_RAW = -1  # the split-K partial sums
_GEMV_ROWS = 8  # most rows of the GEMV
CHUNK = 16  # tokens of a chunk of a recurrent layer


def round_up(n: int, to: int) -> int:
    return -(-n // to) * to


def rms_norm_f32(x: torch.Tensor, weight: torch.Tensor, eps: float, groups: int = 1) -> torch.Tensor:
    from petals_amd.ops import _hip

    # in every library of pre-norm blocks: the one this process serves with
    hip = _hip.first_loaded("hybrid", "recurrent", "scores")
    d = x.shape[-1]
    rows = x.float().reshape(-1, d).contiguous()
    return hip.residual_norm(rows, None, None, weight.float().contiguous(), d, eps, True, 1.0, groups)[:, :d].reshape(x.shape)


def attention_run(batch, heads: int, kv_heads: int) -> int:
    """Rows of a paged attention tile: twice as many where that still fills the chip."""
    return batch.run_tokens(heads // kv_heads, 128 if batch.tokens * heads >= 1 << 16 else 64)


class PackedBlock:
    quant = "none"
    captures = True  # whether the mixer's decoding kernels take its sizes
    mult = 1.0  # factor of what a sublayer adds to the residual

    def __init__(self, block, hip):
        self.hip = hip
        self.spec, self.mlp, self.eps = block.mixer, block.mlp, block.eps
        dtype, dev = block.o.dtype, block.o.device
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"these blocks are served in bfloat16 or float32, not {dtype}")
        self.dtype, self.f32, self.device = dtype, dtype == torch.float32, dev
        self.d = block.config.hidden_size
        self.dp = round_up(self.d, 8)
        self._views = {}  # checkpoint-shaped views of packed weights

    def _finish(self, block) -> None:
        """The feed-forward's two products; frees the block's own weights."""
        if self.mlp is not None:
            ffp = round_up(self.mlp.ff, 8)
            self.w_up, self.w_down = self._zeros(self.dp, ffp), self._zeros(ffp, self.dp)
            self._place(block, "up", self.w_up[: self.d, : self.mlp.ff].t())
            self._place(block, "down", self.w_down[: self.mlp.ff, : self.d].t())
            self.b_up = torch.zeros(ffp, device=self.device)
            self._place(block, "up_bias", self.b_up[: self.mlp.ff])
            self.b_down = self._f32(block, "down_bias")
        self._release(block)

    def _release(self, block) -> None:
        """Frees the block's own weights; all are packed."""
        self.max_gemv_rows = _GEMV_ROWS
        # batches that the engine may capture: only kernels of this library run
        self.max_graph_rows = 0 if self.f32 or not self.captures else self.max_gemv_rows
        self.graph_safe = self.max_graph_rows > 0
        self._no_ws = torch.empty(0, dtype=torch.float32, device=self.device)
        empty = torch.empty(0, dtype=self.dtype, device=self.device)
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
            n += round_up(heads * padded, 8)
        self.w_in = self._zeros(self.dp, n)
        for at, (name, heads, size, padded) in zip(starts, parts):
            heads_view = self.w_in[: self.d, at : at + heads * padded].unflatten(1, (heads, padded))[:, :, :size]
            self._place(block, name, heads_view.permute(1, 2, 0))
        return starts

    # ---------------------------------------------------------------- products

    def _splits(self, w: torch.Tensor) -> int:
        # 64 input rows a wave keeps the loads of a short gemv in flight
        return max(1, min(w.shape[0] // 64, 1024 // (-(-w.shape[1] // 512))))

    def _dense(self, x, w, few: bool, epilogue: int = _EPI_PLAIN_F32, bias=None):
        """x [T, in] (32-bit if few rows or float32, else the weight dtype) @ w [in, out]."""
        if few:
            return self.hip.gemv_bf16(w, x, self._no_ws, None, epilogue, self._splits(w), bias)
        return x @ w

    def _parts(self, x, w):
        """x [T, in] @ w [in, out], as [parts, T, out] to be summed where whole tiles of the
        result (256 x 256) would leave compute units idle: the parts share the inputs."""
        tiles = -(-x.shape[0] // 256) * -(-w.shape[1] // 256)
        parts = 1 if self.f32 else 8
        while parts > 1 and (parts * tiles > 256 or w.shape[0] % (8 * parts) or w.shape[0] < 512 * parts):
            parts //= 2
        if parts == 1:
            return x @ w
        return torch.bmm(x.view(x.shape[0], parts, -1).transpose(0, 1), w.view(parts, -1, w.shape[1]))

    def _add(self, x, y, w, few: bool, bias=None):
        """x += mult (y @ w + bias), for the last product before x is read again."""
        if few:
            self.hip.residual_sum(self._dense(y, w, True, _EPI_RAW), bias, x, self.d, self.mult)
        else:
            self.hip.residual_norm(x, self._parts(y, w), bias, None, self.d, self.eps, True, self.mult)

    def _add_and_norm(self, x, y, w, few: bool, norm):
        """x += mult (y @ w); the norm of the new x, the input of a dense product."""
        if few:
            self._add(x, y, w, True)
            return self.hip.residual_norm(x, None, None, norm, self.d, self.eps, True)
        return self.hip.residual_norm(x, self._parts(y, w), None, norm, self.d, self.eps, self.f32, self.mult)
