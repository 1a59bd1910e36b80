"""Step function of a span of paged blocks.

One call runs the new rows of any number of sequences - portions of prompts and
single decoded tokens together - through all blocks of a span. The handler
(server/handler.py) merges the steps of concurrent sessions into such calls, and
cli/trace_run.py replays recorded steps through it.

When every entry is a single token and the batch is small, the span's kernels
are launched as one captured hipGraph per batch size; positions and page tables
are read from device buffers (paged_cache.StaticDecodeBatch).
"""

from __future__ import annotations

import dataclasses
import os
from typing import Any, Dict, List, Optional, Sequence, Tuple

import torch

from petals_amd.server.paged_cache import PAGE_SIZE, PagedBatch, PagedPool, PagedSequence, StaticDecodeBatch, pages_for

MAX_STEP_TOKENS = 8192  # rows per pass; longer steps are cut into several


@dataclasses.dataclass
class StepEntry:
    """New rows of one sequence. prompts[i], if given, is added to the sequence's
    first positions ahead of block i (deep prompt tuning)."""

    sequence: PagedSequence
    hidden: torch.Tensor  # [n, width]
    start: int
    prompts: Optional[List[Optional[torch.Tensor]]] = None


class SpanEngine:
    def __init__(
        self,
        blocks: Dict[Any, torch.nn.Module],
        pool: PagedPool,
        *,
        max_length: int,
        max_step_tokens: int = MAX_STEP_TOKENS,
    ):
        self.blocks, self.pool, self.device = dict(blocks), pool, pool.device
        self.max_length = max_length
        self.max_step_tokens = max_step_tokens
        self._graphs: Dict[Tuple, _DecodeGraph] = {}

    @staticmethod
    def pool_for(blocks: Sequence[torch.nn.Module], tokens: int, *, dtype, device, max_sequences=None) -> PagedPool:
        widths = {b.layer_idx: b.paged_cache_width() for b in blocks if b.paged_cache_width()}
        states = {b.layer_idx: b.state_shapes() for b in blocks if getattr(b, "state_shapes", dict)()}
        return PagedPool(
            widths, max(1, pages_for(tokens)), dtype=dtype, device=device, max_sequences=max_sequences, states=states
        )

    def check_chain(self, uids: Sequence[Any]) -> None:
        """A chain must contain the owner of every cache it reads, in order."""
        seen = set()
        for uid in uids:
            block = self.blocks[uid]
            if block.source_layer != block.layer_idx and block.source_layer not in seen:
                raise ValueError(
                    f"block {block.layer_idx} reads the cache of block {block.source_layer}: "
                    "both must be in one server's part of the chain"
                )
            seen.add(block.layer_idx)

    @torch.inference_mode()
    def step(self, uids: Sequence[Any], entries: Sequence[StepEntry], pool: Optional[PagedPool] = None) -> List[Any]:
        """Runs the chain `uids` on all entries; returns each entry's output rows
        (or the exception that kept it out of the batch, e.g. a full cache).
        `pool`: where the entries' sequences live (default: the engine's own)."""
        uids = tuple(uids)
        assert all(e.hidden.shape[0] > 0 for e in entries)
        results: List[Any] = [None] * len(entries)
        todo = [(i, 0) for i in range(len(entries))]  # entry, rows done
        while todo:
            batch, later, budget = [], [], self.max_step_tokens
            for i, done in todo:
                n = min(entries[i].hidden.shape[0] - done, budget)
                if n == 0:
                    later.append((i, done))
                    continue
                try:
                    entries[i].sequence.prepare(entries[i].start + done, n)
                except Exception as e:  # noqa: BLE001 - this entry's own failure
                    results[i] = e
                    continue
                budget -= n
                batch.append((i, done, n))
            if batch:
                x, at = self._run(uids, [(entries[i], done, n) for i, done, n in batch], pool or self.pool), 0
                for i, done, n in batch:
                    entries[i].sequence.advance(n)
                    rows = x[at : at + n]
                    results[i] = rows if done == 0 else torch.cat([results[i], rows])
                    at += n
                    if done + n < entries[i].hidden.shape[0]:
                        later.append((i, done + n))
            todo = later
        return results

    def _run(self, uids, parts, pool: PagedPool) -> torch.Tensor:
        hidden = [e.hidden[done : done + n].to(self.device, torch.float32) for e, done, n in parts]
        x = torch.cat(hidden)  # a copy: blocks may update the stream in place
        pages = [e.sequence.pages for e, _, _ in parts]
        starts = [e.start + done for e, done, _ in parts]
        lens = [n for _, _, n in parts]
        slots = [e.sequence.slot for e, _, _ in parts]
        has_prompts = any(e.prompts is not None for e, _, _ in parts)
        if not has_prompts and pool is self.pool and self._graphable(uids, lens):
            key = (uids, len(lens))
            if key not in self._graphs:
                self._graphs[key] = _DecodeGraph(self, uids, len(lens), x, pages, starts)
            return self._graphs[key].step(x, pages, starts, slots)
        batch = PagedBatch(pages, starts, lens, self.device, slots)
        for b, uid in enumerate(uids):
            if has_prompts:
                x = self._add_prompts(x, parts, b)
            x = self.blocks[uid].forward_paged(x, batch, pool)
        return x

    @torch.inference_mode()
    def forward(
        self, uids: Sequence[Any], hidden: torch.Tensor, prompts: Optional[Sequence[Optional[torch.Tensor]]] = None
    ) -> torch.Tensor:
        """Stateless pass over whole sequences [B, S, width] (a scratch pool holds
        their state meanwhile). prompts[i]: [B, pre, width] or None for block i."""
        self.check_chain(uids)
        b, s, _ = hidden.shape
        scratch = self.pool_for(
            [self.blocks[u] for u in uids], b * pages_for(s) * PAGE_SIZE, dtype=self.pool.dtype, device=self.device,
            max_sequences=b,
        )
        entries = [
            StepEntry(
                scratch.open(), hidden[i], 0,
                None if prompts is None else [None if p is None else p[i] for p in prompts],
            )
            for i in range(b)
        ]
        out = self.step(uids, entries, scratch)
        for r in out:
            if isinstance(r, BaseException):
                raise r
        return torch.stack(out)

    def units(self, uids: Sequence[Any]) -> List[List[Any]]:
        """The chain in the smallest runs that share no state with each other."""
        runs: List[List[Any]] = []
        for uid in uids:
            source = self.blocks[uid].source_layer
            keep = len(runs)
            for i, run in enumerate(runs):
                if any(self.blocks[u].layer_idx == source for u in run):
                    keep = i
                    break
            runs[keep:] = [[u for run in runs[keep:] for u in run] + [uid]]
        return runs

    @staticmethod
    def _add_prompts(x, parts, block: int) -> torch.Tensor:
        x, at = x.clone(), 0
        for e, done, n in parts:
            p = e.prompts[block] if e.prompts is not None else None
            if p is not None and done < p.shape[0]:
                stop = min(n, p.shape[0] - done)
                x[at : at + stop, : p.shape[1]] += p[done : done + stop].to(x.device, x.dtype)
            at += n
        return x

    def _graphable(self, uids, lens) -> bool:
        return (
            self.device.type == "cuda"
            and all(n == 1 for n in lens)
            and not os.environ.get("PETALS_AMD_NO_GRAPHS")
            and all(
                self.blocks[u]._fast is not None and len(lens) <= self.blocks[u]._fast.max_graph_rows for u in uids
            )
        )


class _DecodeGraph:
    """The span's kernels for `size` single-token rows, captured once."""

    def __init__(self, engine: SpanEngine, uids, size: int, x: torch.Tensor, pages, starts):
        from petals_amd.utils.graphs import GraphedCallable

        width = min(pages_for(engine.max_length), engine.pool.num_pages)
        self.width = width
        self.batch = StaticDecodeBatch(size, width, engine.device)
        self.x = torch.empty(size, x.shape[1], dtype=torch.float32, device=engine.device)
        # the warm-up runs write the cache of the step that is about to run, which
        # writes it again, and no sequence's recurrent state
        self._load(x, pages, starts, [engine.pool.scratch_slot] * size)

        def span_fn():
            h = self.x
            for uid in uids:
                h = engine.blocks[uid].forward_paged(h, self.batch, engine.pool)
            return h

        self.graph = GraphedCallable(span_fn, [])

    def _load(self, x, pages, starts, slots) -> None:
        longest = max(len(p) for p in pages)
        if longest > self.width:
            raise ValueError(f"a sequence holds {longest} pages, the step graph was made for {self.width}")
        self.x.copy_(x)
        self.batch.load(pages, starts, slots)

    def step(self, x: torch.Tensor, pages, starts, slots) -> torch.Tensor:
        self._load(x, pages, starts, slots)
        return self.graph.replay().clone()
