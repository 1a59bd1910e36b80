"""A whole model of a paged family in one process: the client's embedding, norm
and head around one SpanEngine that hosts every block.

The parts are those of the swarm - same loader, blocks, page pool, step function
and client modules - without the network between them. Used by cli/trace_run.py
and by bench.py.
"""

from __future__ import annotations

import dataclasses
from typing import Dict, List, Optional, Sequence

import torch

from petals_amd.server.from_pretrained import load_pretrained_block
from petals_amd.server.paged_cache import PagedSequence
from petals_amd.server.span_engine import SpanEngine, StepEntry


@dataclasses.dataclass
class Request:
    """Next tokens of one request and the places among them whose logits are wanted."""

    id: str
    tokens: List[int]
    want: List[int]


class LocalEngine:
    def __init__(
        self,
        model_dir: str,
        *,
        dtype: torch.dtype,
        device: torch.device,
        max_tokens: int,
        max_requests: Optional[int] = None,
    ):
        from petals_amd.utils.auto_config import AutoDistributedModelForCausalLM

        self.device, self.dtype = torch.device(device), dtype
        self.model = AutoDistributedModelForCausalLM.from_pretrained(model_dir, standalone=True)
        self.model = self.model.to(device=self.device, dtype=dtype).eval()
        self.config = self.model.config
        blocks = {
            i: load_pretrained_block(model_dir, self.config, i, torch_dtype=dtype, device=self.device)
            for i in range(self.config.num_blocks)
        }
        if not all(getattr(b, "paged", False) for b in blocks.values()):
            raise ValueError(f"model_type {self.config.model_type!r} has no paged blocks")
        pool = SpanEngine.pool_for(
            list(blocks.values()), max_tokens, dtype=dtype, device=self.device, max_sequences=max_requests
        )
        self.engine = SpanEngine(blocks, pool, max_length=max_tokens)
        self.uids = tuple(blocks)
        self.engine.check_chain(self.uids)
        self.live: Dict[str, PagedSequence] = {}

    @torch.inference_mode()
    def hidden(self, requests: Sequence[Request]) -> List[torch.Tensor]:
        """Residual stream behind the last block, one [n, width] per request."""
        entries = []
        for r in requests:
            if r.id not in self.live:
                self.live[r.id] = self.engine.pool.open()
            seq = self.live[r.id]
            ids = torch.tensor(r.tokens, dtype=torch.long).to(self.device)
            x = self.model.transformer._prepare_embeds(self.model.transformer._embed(ids))
            entries.append(StepEntry(seq, x, seq.length))
        out = self.engine.step(self.uids, entries)
        for r in out:
            if isinstance(r, BaseException):
                raise r
        return out

    @torch.inference_mode()
    def step(self, requests: Sequence[Request]) -> torch.Tensor:
        """Runs one batch; returns the wanted logits [wanted, vocab], 32-bit."""
        hidden = self.hidden(requests)
        rows = [h[r.want] for h, r in zip(hidden, requests) if r.want]
        if not rows:
            return torch.empty(0, self.config.vocab_size)
        return self.model.lm_head(self.model.transformer.norm(torch.cat(rows))).float().cpu()

    def end(self, request_id: str) -> None:
        self.live.pop(request_id).close()
