"""Paged attention-state pool: one set of fixed-size pages for all sequences.

Per-session contiguous tensors (server/memory_cache.py TensorDescriptor) suit
families whose step is one session wide. Families with ``paged`` blocks keep
their per-token state in pages instead, so that rows of many sequences -
portions of prompts beside single decoded tokens - run as one ragged batch:

  PagedPool      the pages of every cache-owning layer, a free list, reference
                 counts (beam hypotheses share full pages; a shared page is
                 copied when it is about to be written)
  PagedSequence  one sequence's page list and length; grows page by page,
                 rolls back, closes
  PageDescriptor reserves a session's worst case from MemoryCache's byte budget
                 (same FIFO queueing and timeouts as tensor caches)
  PagedBatch     the rows of one step: positions, owners and page tables
"""

from __future__ import annotations

import threading
from typing import Dict, List, Optional, Sequence, Tuple

import torch

from petals_amd.server.memory_cache import AllocationFailed
from petals_amd.utils.misc import get_size_in_bytes

PAGE_SIZE = 64  # tokens


def pages_for(tokens: int) -> int:
    return -(-tokens // PAGE_SIZE)


class PagedPool:
    def __init__(
        self,
        layer_widths: Dict[int, int],
        num_pages: int,
        *,
        dtype: torch.dtype,
        device: torch.device,
        max_sequences: Optional[int] = None,
    ):
        self.num_pages, self.dtype, self.device = num_pages, dtype, torch.device(device)
        self.max_sequences = max_sequences
        self._layers = {
            layer: torch.zeros(num_pages, PAGE_SIZE, width, dtype=dtype, device=device)
            for layer, width in layer_widths.items()
        }
        self.bytes_per_page = sum(layer_widths.values()) * PAGE_SIZE * get_size_in_bytes(dtype)
        self._free = list(range(num_pages - 1, -1, -1))
        self._refs = [0] * num_pages
        self._lock = threading.Lock()
        self.live_sequences = 0

    @property
    def free_pages(self) -> int:
        return len(self._free)

    def layer(self, layer: int) -> torch.Tensor:
        """[pages, page size, width] of one cache-owning layer."""
        try:
            return self._layers[layer]
        except KeyError:
            raise ValueError(f"the cache of block {layer} is not in this server's span") from None

    def open(self) -> "PagedSequence":
        with self._lock:
            if self.max_sequences is not None and self.live_sequences >= self.max_sequences:
                raise AllocationFailed(f"all {self.max_sequences} sequence slots are in use")
            self.live_sequences += 1
        return PagedSequence(self)

    # ------------------------------------------------------ page accounting

    def _take(self, n: int) -> List[int]:
        with self._lock:
            if n > len(self._free):
                raise AllocationFailed(f"{n} pages needed, {len(self._free)} of {self.num_pages} free")
            taken = [self._free.pop() for _ in range(n)]
            for p in taken:
                self._refs[p] = 1
            return taken

    def _share(self, pages: Sequence[int]) -> None:
        with self._lock:
            for p in pages:
                self._refs[p] += 1

    def _release(self, pages: Sequence[int]) -> None:
        with self._lock:
            for p in pages:
                self._refs[p] -= 1
                if self._refs[p] == 0:
                    self._free.append(p)

    def _copy(self, src: int, dst: int) -> None:
        for t in self._layers.values():
            t[dst].copy_(t[src])

    def reorder(self, sequences: Sequence["PagedSequence"], parents: Sequence[int]) -> None:
        """Beam search: sequence i continues hypothesis parents[i]. Pages are
        shared, not copied; PagedSequence.prepare copies on write."""
        if list(parents) == list(range(len(sequences))):
            return
        new = [(list(sequences[p].pages), sequences[p].length) for p in parents]
        for pages, _ in new:
            self._share(pages)
        for seq, (pages, length) in zip(sequences, new):
            self._release(seq.pages)
            seq.pages, seq.length = pages, length


class PagedSequence:
    def __init__(self, pool: PagedPool):
        self.pool = pool
        self.pages: List[int] = []
        self.length = 0  # tokens whose state is valid
        self._open = True

    def prepare(self, start: int, n: int) -> None:
        """Make positions [start, start + n) writable. A start before the
        current length rolls back: the state behind it is dropped."""
        if not self._open:
            raise RuntimeError("the sequence is closed")
        if start > self.length:
            raise ValueError(f"position {start} is ahead of the cache ({self.length} tokens)")
        pool = self.pool
        need = pages_for(start + n)
        if need > len(self.pages):
            self.pages += pool._take(need - len(self.pages))
        elif need < len(self.pages):
            pool._release(self.pages[need:])
            del self.pages[need:]
        self.length = start
        for i in range(start // PAGE_SIZE, need):
            if pool._refs[self.pages[i]] > 1:
                (fresh,) = pool._take(1)
                pool._copy(self.pages[i], fresh)
                pool._release([self.pages[i]])
                self.pages[i] = fresh

    def advance(self, n: int) -> None:
        self.length += n

    def close(self) -> None:
        if self._open:
            self._open = False
            self.pool._release(self.pages)
            self.pages, self.length = [], 0
            with self.pool._lock:
                self.pool.live_sequences -= 1


class PageDescriptor:
    """MemoryCache descriptor of a session of `batch_size` paged sequences."""

    def __init__(self, pool: PagedPool, batch_size: int, max_length: int):
        self.pool, self.batch_size = pool, batch_size
        self.nbytes = batch_size * pages_for(max_length) * pool.bytes_per_page

    def allocate(self, device) -> List[PagedSequence]:
        return [self.pool.open() for _ in range(self.batch_size)]

    def release(self, sequences: List[PagedSequence]) -> None:
        for s in sequences:
            s.close()


class PagedBatch:
    """Rows of one step, grouped by sequence: sequence s brings rows
    [offsets[s], offsets[s+1]) at positions starts[s], starts[s]+1, ..."""

    def __init__(self, pages: List[List[int]], starts: List[int], lens: List[int], device: torch.device):
        self.pages, self.starts, self.lens = pages, starts, lens
        self.tokens = sum(lens)
        self.device = torch.device(device)
        self.max_end = max(s + n for s, n in zip(starts, lens))
        self._tiles: Dict[int, torch.Tensor] = {}
        if self.device.type == "cuda":
            self._upload()

    @property
    def decode_only(self) -> bool:
        return all(n == 1 for n in self.lens)

    def row_ranges(self) -> List[Tuple[int, int]]:
        ranges, at = [], 0
        for n in self.lens:
            ranges.append((at, at + n))
            at += n
        return ranges

    def _host_ints(self, values: List[int]) -> torch.Tensor:
        return torch.tensor(values, dtype=torch.int32, pin_memory=True)

    def _upload(self) -> None:
        """One int32 copy to the device: pos [T], owner [T], tables [S, width]."""
        t, width = self.tokens, max(len(p) for p in self.pages)
        flat: List[int] = []
        for s, n in zip(self.starts, self.lens):
            flat.extend(range(s, s + n))
        for i, n in enumerate(self.lens):
            flat.extend([i] * n)
        for p in self.pages:
            flat.extend(p)
            flat.extend([0] * (width - len(p)))
        dev = self._host_ints(flat).to(self.device, non_blocking=True)
        self.pos, self.owner = dev[:t], dev[t : 2 * t]
        self.tables = dev[2 * t :].view(len(self.pages), width)

    def run_tokens(self, heads: int) -> int:
        """Rows that share one attention tile: as many as give about 64
        (row, head) pairs."""
        return 1 if self.decode_only else max(1, 64 // heads)

    def tiles(self, rows: int) -> torch.Tensor:
        """[n, 2] int32 (first row, row count): the batch's rows in runs of at
        most `rows`, no run crossing a sequence."""
        if rows not in self._tiles:
            flat: List[int] = []
            for lo, hi in self.row_ranges():
                for r in range(lo, hi, rows):
                    flat += [r, min(rows, hi - r)]
            self._tiles[rows] = self._host_ints(flat).to(self.device, non_blocking=True).view(-1, 2)
        return self._tiles[rows]


class StaticDecodeBatch(PagedBatch):
    """One row for each of `size` sequences in device buffers that keep their
    addresses, so that a captured graph replays with new positions and pages."""

    def __init__(self, size: int, width: int, device: torch.device):
        self.lens, self.tokens = [1] * size, size
        self.device = torch.device(device)
        self.starts, self.pages = [0] * size, [[0]] * size
        self.max_end = width * PAGE_SIZE
        self._tiles = {}
        self.pos = torch.zeros(size, dtype=torch.int32, device=device)
        self.owner = torch.arange(size, dtype=torch.int32, device=device)
        self.tables = torch.zeros(size, width, dtype=torch.int32, device=device)
        self._uploaded: List[Optional[List[int]]] = [None] * size
        self.tiles(1)

    def load(self, pages: List[List[int]], starts: List[int]) -> None:
        self.pos.copy_(self._host_ints(starts), non_blocking=True)
        for i, p in enumerate(pages):
            if self._uploaded[i] != p:
                self.tables[i, : len(p)].copy_(self._host_ints(p), non_blocking=True)
                self._uploaded[i] = list(p)
