"""Paged cache, state slots and ragged batches.

A ragged batch runs any mix of requests in one forward: portions of prompts
beside single decoded tokens, flattened to rows.  What requests keep between
steps lives in two kinds of shared storage:

  * rows of a paged layer (per token), in pages of ``PAGE`` tokens;
  * the state of a recurrent layer and the last inputs of short convolutions
    (per request), in slots.

Pages and slots are handed out when a request is admitted or grows and come
back when it ends.  Nothing is cleared in between: attention reads only rows
below a request's length, and a request at position 0 starts from a zero state
whatever its slot holds.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, Hashable, List, Optional, Sequence, Tuple

import numpy as np
import torch

PAGE = 64    # tokens per cache page
SHORT = 16   # portions up to this long take the decode kernels
CHUNK = 64   # tokens per chunk of the chunked recurrence
QTILE = 128  # query rows per block of the expanded attention
SPAN = 128   # tokens that one pass of the selective scan takes in sequence


class CacheFull(RuntimeError):
    """No page or slot is free."""


@dataclass
class RowSpec:
    """A paged layer: ``width`` elements per token."""
    width: int


@dataclass
class StateSpec:
    """A recurrent layer: fp32 state [heads, dim, vdim] and the last inputs
    of a short convolution [channels, history] (no channels: none)."""
    heads: int
    dim: int
    vdim: int
    channels: int = 0
    history: int = 0


@dataclass
class HistorySpec:
    """The last ``history`` input rows of a causal convolution over time."""
    channels: int
    history: int


@dataclass
class LayerSpec:
    """A layer that keeps more than its mixer's storage: besides ``mix`` (a
    RowSpec, a StateSpec or None) the histories of its convolutions by name."""
    mix: Optional[object]
    histories: Dict[str, HistorySpec]


class LayerStore:
    """Storage of one layer: ``rows`` or ``state`` + ``conv``, and
    ``histories`` [slots, history, channels]."""

    __slots__ = ("spec", "rows", "state", "conv", "histories")

    def __init__(self, spec, n_pages: int, n_slots: int, dtype, device):
        histories = {}
        if isinstance(spec, LayerSpec):
            spec, histories = spec.mix, spec.histories
        self.spec = spec
        self.rows = self.state = self.conv = None
        self.histories: Dict[str, torch.Tensor] = {
            name: torch.empty(n_slots, h.history, h.channels, dtype=dtype,
                              device=device)
            for name, h in histories.items()}
        if isinstance(spec, RowSpec):
            self.rows = torch.empty(n_pages * PAGE, spec.width, dtype=dtype,
                                    device=device)
        elif spec is not None:
            self.state = torch.empty(n_slots, spec.heads, spec.dim, spec.vdim,
                                     dtype=torch.float32, device=device)
            if spec.channels:
                self.conv = torch.empty(n_slots, spec.channels, spec.history,
                                        dtype=dtype, device=device)

    def per_slot(self) -> List[torch.Tensor]:
        """What moves on with every token instead of being kept per token."""
        found = [self.state, self.conv, *self.histories.values()]
        return [t for t in found if t is not None and t.numel()]

    def grow_rows(self, n_pages: int):
        if self.rows is None:
            return
        rows = torch.empty(n_pages * PAGE, self.spec.width,
                           dtype=self.rows.dtype, device=self.rows.device)
        rows[: self.rows.shape[0]] = self.rows
        self.rows = rows


@dataclass
class Held:
    """What one live request holds."""
    slot: int
    pages: List[int]
    length: int = 0


class PagedState:
    """Cache and state manager of one stage model."""

    def __init__(self, specs: Sequence, max_tokens: int, max_requests: int,
                 dtype: torch.dtype, device):
        self.n_pages = (max_tokens + PAGE - 1) // PAGE
        self.n_slots = max_requests
        self.device = torch.device(device)
        self.dtype = dtype
        # a layer that keeps nothing of its own has spec None
        self.layers: List[Optional[LayerStore]] = [
            None if s is None else
            LayerStore(s, self.n_pages, self.n_slots, dtype, device)
            for s in specs]
        self._free_pages = list(range(self.n_pages - 1, -1, -1))
        self._free_slots = list(range(self.n_slots - 1, -1, -1))
        self.live: Dict[Hashable, Held] = {}

    @property
    def free_tokens(self) -> int:
        return len(self._free_pages) * PAGE

    @property
    def free_slots(self) -> int:
        return len(self._free_slots)

    def admit(self, rid: Hashable) -> Held:
        if rid in self.live:
            raise ValueError(f"request {rid!r} is live already")
        if not self._free_slots:
            raise CacheFull(f"all {self.n_slots} request slots are in use")
        held = Held(self._free_slots.pop(), [])
        self.live[rid] = held
        return held

    def reserve(self, rid: Hashable, length: int):
        """Pages for ``length`` tokens in all; takes none if too few are free."""
        held = self.live[rid]
        need = (length + PAGE - 1) // PAGE - len(held.pages)
        if need > len(self._free_pages):
            raise CacheFull(f"request {rid!r} needs {need} more pages, "
                            f"{len(self._free_pages)} are free")
        for _ in range(need):
            held.pages.append(self._free_pages.pop())

    def release(self, rid: Hashable):
        held = self.live.pop(rid)
        self._free_pages.extend(reversed(held.pages))
        self._free_slots.append(held.slot)

    def grow(self, n_pages: int):
        """More pages; what is stored stays where it is."""
        if n_pages <= self.n_pages:
            return
        for layer in self.layers:
            if layer is not None:
                layer.grow_rows(n_pages)
        self._free_pages[:0] = range(n_pages - 1, self.n_pages - 1, -1)
        self.n_pages = n_pages


class RaggedBatch:
    """Who runs what in one forward: requests, portions, places.

    Requests are ordered short portions first (``order`` maps back), so that
    short and long tokens are two slices of every activation.  All arrays the
    kernels read travel in one int32 copy.
    """

    def __init__(self, portions: Sequence[Tuple[Held, int]], device,
                 max_keys: int = 0):
        """portions: (what the request holds, number of new tokens)."""
        lens = [n for _, n in portions]
        self.order = sorted(range(len(portions)),
                            key=lambda i: lens[i] > SHORT)
        held = [portions[i][0] for i in self.order]
        n = np.array([lens[i] for i in self.order], dtype=np.int32)
        pos0 = np.array([h.length for h in held], dtype=np.int32)
        E = len(held)
        self.n_requests = E
        self.n_short = int((n <= SHORT).sum())
        self.n_long = E - self.n_short
        cu = np.zeros(E + 1, dtype=np.int32)
        np.cumsum(n, out=cu[1:])
        self.n_tokens = int(cu[E])
        self.short_tokens = int(cu[self.n_short])
        self.max_len = int(n.max())
        self.max_short = int(n[: self.n_short].max()) if self.n_short else 0
        ends = pos0 + n
        self.max_pos = int(ends.max())
        self.max_keys = max(max_keys, self.max_pos)
        P = max(1, max(len(h.pages) for h in held))
        pages = np.zeros((E, P), dtype=np.int32)
        for e, h in enumerate(held):
            pages[e, : len(h.pages)] = h.pages
        tok_entry = np.repeat(np.arange(E, dtype=np.int32), n)
        tok_pos = (np.arange(self.n_tokens, dtype=np.int32)
                   - cu[tok_entry] + pos0[tok_entry]).astype(np.int32)
        parts = {
            "cu": cu, "pos0": pos0,
            "slots": np.array([h.slot for h in held], dtype=np.int32),
            "tok_pos": tok_pos, "tok_entry": tok_entry, "pages": pages,
        }
        self.key_rows = 0
        if self.n_long:
            nl, pl = n[self.n_short:], pos0[self.n_short:]
            el = ends[self.n_short:]
            kpad = (el + PAGE - 1) // PAGE * PAGE
            cuk = np.zeros(self.n_long + 1, dtype=np.int32)
            np.cumsum(kpad, out=cuk[1:])
            self.key_rows = int(cuk[-1])
            blocks, fills, tiles, chunks, chunk_cu = [], [], [], [], [0]
            spans, span_cu = [], [0]
            for j in range(self.n_long):
                e = self.n_short + j
                for b in range(kpad[j] // PAGE):
                    blocks.append((pages[e, b], cuk[j] + b * PAGE,
                                   min(PAGE, el[j] - b * PAGE)))
                for b in range(pl[j] // PAGE, kpad[j] // PAGE):
                    t = cu[e] - pl[j] + b * PAGE  # token of the first slot
                    fills.append((pages[e, b], t, max(0, pl[j] - b * PAGE),
                                  min(PAGE, el[j] - b * PAGE)))
                for q0 in range(0, nl[j], QTILE):
                    tiles.append((-(pl[j] + q0), e, q0))
                for c in range(0, nl[j], CHUNK):
                    chunks.append((cu[e] + c, min(CHUNK, nl[j] - c)))
                chunk_cu.append(len(chunks))
                for c in range(0, nl[j], SPAN):
                    spans.append((cu[e] + c, min(SPAN, nl[j] - c), e,
                                  c + SPAN >= nl[j]))
                span_cu.append(len(spans))
            tiles.sort()  # most keys first
            parts.update(
                cuk=cuk, blocks=np.array(blocks, dtype=np.int32),
                fills=np.array(fills, dtype=np.int32),
                tiles=np.array(tiles, dtype=np.int32)[:, 1:],
                chunks=np.array(chunks, dtype=np.int32),
                chunk_cu=np.array(chunk_cu, dtype=np.int32),
                # (first token, tokens, request, whether the portion ends)
                spans=np.array(spans, dtype=np.int32),
                span_cu=np.array(span_cu, dtype=np.int32))
        flat = np.concatenate([np.ascontiguousarray(a).reshape(-1)
                               for a in parts.values()])
        dev = torch.from_numpy(flat).to(device)
        off = 0
        for name, a in parts.items():
            setattr(self, name, dev[off: off + a.size].view(a.shape))
            off += a.size
        self.host = [(int(cu[e]), int(n[e]), int(pos0[e]), held[e])
                     for e in range(E)]

    def advance(self):
        """Turn a batch of single tokens into the next one, on the device;
        pages must not have grown since."""
        self.tok_pos.add_(1)
        self.pos0.add_(1)
        self.max_pos += 1
        self.max_keys = max(self.max_keys, self.max_pos)
        self.host = [(s, n, p + 1, h) for s, n, p, h in self.host]


class RaggedCache:
    """The batch-of-equals view of PagedState that the pipeline loops drive:
    B sequences of equal length, growing together (see ops.kvcache.KVCache,
    whose lifecycle — offset, ensure_capacity, graph_pos, reset — it keeps).
    """

    GROW = 1024

    def __init__(self, specs: Sequence, batch_size: int, dtype, device):
        self.batch_size = batch_size
        self.offset = 0
        self._graph_pos: Optional[torch.Tensor] = None
        self.state = PagedState(specs, 0, batch_size, dtype, device)
        self.held = [self.state.admit(b) for b in range(batch_size)]
        self.capacity = 0
        self._decode: Optional[RaggedBatch] = None
        # one batch per captured position; a graph reads its arrays for as
        # long as it may be replayed, so they are kept
        self._graph_batches: List[Tuple[torch.Tensor, RaggedBatch]] = []

    def ensure_capacity(self, cap: int):
        if cap <= self.capacity:
            return
        cap = (cap + self.GROW - 1) // self.GROW * self.GROW
        self.state.grow(self.batch_size * cap // PAGE)
        for b in range(self.batch_size):
            self.state.reserve(b, cap)
        self.capacity = cap
        self._decode = None

    @property
    def graph_pos(self):
        return self._graph_pos

    @graph_pos.setter
    def graph_pos(self, pos):
        if pos is not None and self._graph_batch(pos) is None:
            # a decode batch of its own, whose places follow the device
            # position; lengths are sized for the whole capacity
            self._graph_batches.append((pos, RaggedBatch(
                [(h, 1) for h in self.held], self.state.device,
                max_keys=self.capacity)))
        self._graph_pos = pos

    def _graph_batch(self, pos: torch.Tensor) -> Optional[RaggedBatch]:
        """The batch a graph with this position was captured on."""
        for p, batch in self._graph_batches:
            if p is pos:
                return batch
        return None

    def next_batch(self, T: int) -> RaggedBatch:
        """The batch of the next T tokens of every sequence."""
        if self._graph_pos is not None:
            if T != 1:
                raise ValueError("a captured decode step has one token")
            b = self._graph_batch(self._graph_pos)
            b.tok_pos.copy_(self._graph_pos.expand(self.batch_size))
            b.pos0.copy_(b.tok_pos)
            b.max_pos = self.capacity
            return b
        self.ensure_capacity(self.offset + T)
        d = self._decode
        if T == 1 and d is not None and d.max_pos == self.offset:
            d.advance()
        else:
            d = RaggedBatch([(h, T) for h in self.held], self.state.device)
        self._decode = d if T == 1 else None
        self.offset += T
        for h in self.held:
            h.length = self.offset
        return d

    def trim(self, n: int):
        """Go back to the first n tokens of every sequence."""
        if not 0 <= n <= self.offset:
            raise ValueError(f"trim({n}) outside [0, {self.offset}]")
        self.offset = n
        self._graph_pos = None
        self._decode = None
        for h in self.held:
            h.length = n

    def reset(self):
        self.trim(0)


class RaggedLayerCache:
    """One layer's handle on a RaggedCache, with KVCache's interface."""

    def __init__(self, shared: RaggedCache, layer: int):
        self.shared = shared
        self.layer = layer

    @property
    def trimmable(self) -> bool:
        """What is kept per slot cannot be rolled back to a shorter prefix;
        rows can."""
        return all(s is None or not s.per_slot()
                   for s in self.shared.state.layers)

    batch_size = property(lambda self: self.shared.batch_size)
    offset = property(lambda self: self.shared.offset)
    capacity = property(lambda self: self.shared.capacity)

    @property
    def graph_pos(self):
        return self.shared.graph_pos

    @graph_pos.setter
    def graph_pos(self, pos):
        self.shared.graph_pos = pos

    def _store(self) -> Optional[LayerStore]:
        return self.shared.state.layers[self.layer]

    def keys_buffer(self) -> Optional[torch.Tensor]:
        """The buffer a captured graph aliases; layers without one of their
        own answer with the first layer that has one."""
        if self.shared.capacity == 0:
            return None
        for s in (self._store(), *self.shared.state.layers):
            if s is not None and (s.rows is not None or s.state is not None):
                return s.rows if s.rows is not None else s.state
        return None

    def ensure_capacity(self, cap: int, batch: Optional[int] = None):
        if batch is not None and batch != self.batch_size:
            raise ValueError(f"cache batch mismatch: {self.batch_size} vs {batch}")
        self.shared.ensure_capacity(cap)

    def snapshot(self):
        s = self._store()
        return [] if s is None else [t.clone() for t in s.per_slot()]

    def restore(self, snap):
        if snap:
            for t, kept in zip(self._store().per_slot(), snap):
                t.copy_(kept)

    def trim(self, n: int):
        if n not in (0, self.shared.offset) and not self.trimmable:
            raise ValueError("a recurrent state has no shorter prefix to go "
                             "back to")
        self.shared.trim(n)

    def reset(self):
        self.shared.reset()
