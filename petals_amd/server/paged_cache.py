"""Paged attention-state pool: one set of fixed-size pages for all sequences.

Per-session contiguous tensors (server/memory_cache.py TensorDescriptor) suit
families whose step is one session wide. Families with ``paged`` blocks keep
their per-token state in pages instead, so that rows of many sequences -
portions of prompts beside single decoded tokens - run as one ragged batch:

  PagedPool      the pages of every cache-owning layer, a free list, reference
                 counts (beam hypotheses share full pages; a shared page is
                 copied when it is about to be written); and, for recurrent
                 layers, one state slot per sequence
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
DEFAULT_SLOTS = 64  # sequences of a pool with recurrent state, if nothing else is said


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
        states: Optional[Dict[int, Dict[str, Tuple[int, ...]]]] = None,
    ):
        """states: recurrent layer -> {name: shape of one sequence's 32-bit state}.
        A slot is not cleared when it is taken: the state of a sequence at
        position 0 is zero whatever the slot holds."""
        self.num_pages, self.dtype, self.device = num_pages, dtype, torch.device(device)
        self.recurrent = bool(states)
        if self.recurrent and max_sequences is None:
            max_sequences = DEFAULT_SLOTS
        self.max_sequences = max_sequences
        self._layers = {
            layer: torch.zeros(num_pages, PAGE_SIZE, width, dtype=dtype, device=device)
            for layer, width in layer_widths.items()
        }
        self.bytes_per_page = sum(layer_widths.values()) * PAGE_SIZE * get_size_in_bytes(dtype)
        slots = max_sequences if self.recurrent else 0
        self._states = {
            layer: {name: torch.zeros(slots + 1, *shape, device=device) for name, shape in shapes.items()}
            for layer, shapes in (states or {}).items()
        }
        self.bytes_per_sequence = sum(4 * t[0].numel() for s in self._states.values() for t in s.values())
        self.scratch_slot = slots  # belongs to no sequence
        self._free_slots = list(range(slots - 1, -1, -1))
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

    def state(self, layer: int) -> Dict[str, torch.Tensor]:
        """name -> [slots + 1, ...] of one recurrent layer."""
        try:
            return self._states[layer]
        except KeyError:
            raise ValueError(f"the state of block {layer} is not in this server's span") from None

    @property
    def total_bytes(self) -> int:
        return self.num_pages * self.bytes_per_page + self.scratch_slot * self.bytes_per_sequence

    def can_open(self, n: int) -> bool:
        return self.max_sequences is None or self.live_sequences + n <= self.max_sequences

    def open(self) -> "PagedSequence":
        with self._lock:
            if not self.can_open(1):
                raise AllocationFailed(f"all {self.max_sequences} sequence slots are in use")
            self.live_sequences += 1
            slot = self._free_slots.pop() if self.recurrent else 0
        return PagedSequence(self, slot)

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
        if self.recurrent:
            own = torch.tensor([s.slot for s in sequences], device=self.device)
            source = own[torch.as_tensor(list(parents), device=self.device)]
            for tensors in self._states.values():
                for t in tensors.values():
                    t[own] = t[source]


class PagedSequence:
    def __init__(self, pool: PagedPool, slot: int = 0):
        self.pool, self.slot = pool, slot
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
        if self.pool.recurrent and start not in (0, self.length):
            raise ValueError(f"the state behind {self.length} tokens cannot go back to {start}; replay from 0")
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
                if self.pool.recurrent:
                    self.pool._free_slots.append(self.slot)


class PageDescriptor:
    """MemoryCache descriptor of a session of `batch_size` paged sequences."""

    def __init__(self, pool: PagedPool, batch_size: int, max_length: int):
        self.pool, self.batch_size = pool, batch_size
        self.nbytes = batch_size * (pages_for(max_length) * pool.bytes_per_page + pool.bytes_per_sequence)

    def ready(self) -> bool:
        return self.pool.can_open(self.batch_size)

    def allocate(self, device) -> List[PagedSequence]:
        return [self.pool.open() for _ in range(self.batch_size)]

    def release(self, sequences: List[PagedSequence]) -> None:
        for s in sequences:
            s.close()


class PagedBatch:
    """Rows of one step, grouped by sequence: sequence s brings rows
    [offsets[s], offsets[s+1]) at positions starts[s], starts[s]+1, ... and its
    recurrent state is in slot slots[s]."""

    def __init__(
        self,
        pages: List[List[int]],
        starts: List[int],
        lens: List[int],
        device: torch.device,
        slots: Optional[List[int]] = None,
    ):
        self.pages, self.starts, self.lens = pages, starts, lens
        self.slots = [0] * len(lens) if slots is None else slots
        self.tokens = sum(lens)
        self.device = torch.device(device)
        self.max_end = max(s + n for s, n in zip(starts, lens))
        self._tiles: Dict[int, torch.Tensor] = {}
        self._chunks: Dict[int, torch.Tensor] = {}
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
        """One int32 copy to the device: pos [T], owner [T], slot [S], tables [S, width]."""
        t, width = self.tokens, max(len(p) for p in self.pages)
        flat: List[int] = []
        for s, n in zip(self.starts, self.lens):
            flat.extend(range(s, s + n))
        for i, n in enumerate(self.lens):
            flat.extend([i] * n)
        flat.extend(self.slots)
        for p in self.pages:
            flat.extend(p)
            flat.extend([0] * (width - len(p)))
        dev = self._host_ints(flat).to(self.device, non_blocking=True)
        self.pos, self.owner = dev[:t], dev[t : 2 * t]
        self.slot = dev[2 * t : 2 * t + len(self.slots)]
        self.tables = dev[2 * t + len(self.slots) :].view(len(self.pages), width)

    def run_tokens(self, heads: int, rows: int = 64) -> int:
        """Rows that share one attention tile: as many as give about `rows`
        (row, head) pairs."""
        return 1 if self.decode_only else max(1, rows // heads)

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

    def chunk_bounds(self, rows: int) -> torch.Tensor:
        """[S + 1] int32: tiles(rows)[bounds[s] : bounds[s + 1]] are sequence s's."""
        if rows not in self._chunks:
            bounds = [0]
            for n in self.lens:
                bounds.append(bounds[-1] - (-n // rows))
            self._chunks[rows] = self._host_ints(bounds).to(self.device, non_blocking=True)
        return self._chunks[rows]


class StaticDecodeBatch(PagedBatch):
    """One row for each of `size` sequences in device buffers that keep their
    addresses, so that a captured graph replays with new positions and pages."""

    def __init__(self, size: int, width: int, device: torch.device):
        self.lens, self.tokens = [1] * size, size
        self.device = torch.device(device)
        self.starts, self.pages = [0] * size, [[0]] * size
        self.max_end = width * PAGE_SIZE
        self._tiles, self._chunks = {}, {}
        self.slots = [0] * size
        self.slot = torch.zeros(size, dtype=torch.int32, device=device)
        self.pos = torch.zeros(size, dtype=torch.int32, device=device)
        self.owner = torch.arange(size, dtype=torch.int32, device=device)
        self.tables = torch.zeros(size, width, dtype=torch.int32, device=device)
        self._uploaded: List[Optional[List[int]]] = [None] * size
        self.tiles(1)

    def load(self, pages: List[List[int]], starts: List[int], slots: List[int]) -> None:
        self.pos.copy_(self._host_ints(starts), non_blocking=True)
        if slots != self.slots:
            self.slot.copy_(self._host_ints(slots), non_blocking=True)
            self.slots = list(slots)
        for i, p in enumerate(pages):
            if self._uploaded[i] != p:
                self.tables[i, : len(p)].copy_(self._host_ints(p), non_blocking=True)
                self._uploaded[i] = list(p)
