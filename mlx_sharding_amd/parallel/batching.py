"""Continuous batching: many requests in one forward.

``BatchEngine`` is the step: it admits requests, runs any mix of prompt
portions and single tokens as one ragged batch over a fixed pool of cache pages
and state slots, and gives back what ended.  ``BatchScheduler`` generates with
it: it admits waiting requests while their pages fit, spends a token budget per
step on decoding first and prompts next, and samples with the same rules as
``engine.generate_step``.  ``BatchService`` puts a scheduler behind a thread so
that concurrent callers share its batches.

Works with every stage model that ``supports_ragged`` and owns all layers.
"""

from __future__ import annotations

import queue
import threading
from collections import deque
from dataclasses import dataclass, field
from typing import (Deque, Dict, Generator, Hashable, Iterator, List, Optional,
                    Sequence, Tuple)

import torch

from ..models.base import StageModel
from ..ops.paged import PAGE, CacheFull, RaggedBatch
from .engine import Sampler, SamplingParams

__all__ = ["BatchEngine", "BatchScheduler", "BatchService", "CacheFull",
           "Portion", "Request"]


@dataclass
class Portion:
    """The next tokens of one request, and the places among them whose logits
    are wanted."""
    rid: Hashable
    tokens: Sequence[int]
    want: Sequence[int] = ()


class BatchEngine:
    def __init__(self, model: StageModel, max_tokens: int, max_requests: int):
        if not model.supports_ragged:
            raise ValueError(f"{model.model_type} does not run ragged batches")
        if not (model.shard.is_first and model.shard.is_last):
            raise ValueError("batches run on a model that owns all layers")
        self.model = model
        self.device = next(model.parameters()).device
        self.vocab = model.config.vocab_size
        self.state = model.make_state(max_tokens, max_requests)
        self._last: Optional[RaggedBatch] = None
        self._last_key: Optional[tuple] = None

    @property
    def live(self) -> Sequence[Hashable]:
        return list(self.state.live)

    def length(self, rid: Hashable) -> int:
        return self.state.live[rid].length

    def step(self, portions: Sequence[Portion]) -> torch.Tensor:
        """Run all portions as one batch.  Returns fp32 logits of the wanted
        places, [wanted, vocab], in the order of the portions."""
        if not portions:
            return torch.empty(0, self.vocab, device=self.device)
        state = self.state
        rids = [p.rid for p in portions]
        if len(set(rids)) != len(rids):
            raise ValueError("a request appears twice in one step")
        for p in portions:
            if not len(p.tokens):
                raise ValueError(f"request {p.rid!r}: empty portion")
            if any(not 0 <= int(t) < self.vocab for t in p.tokens):
                raise ValueError(f"request {p.rid!r}: token out of range")
            if any(not 0 <= int(w) < len(p.tokens) for w in p.want):
                raise ValueError(f"request {p.rid!r}: wanted place out of range")
        fresh = [r for r in rids if r not in state.live]
        pages = {r: len(state.live[r].pages) for r in rids if r in state.live}
        try:
            for r in fresh:
                state.admit(r)
            for p in portions:
                state.reserve(p.rid, state.live[p.rid].length + len(p.tokens))
        except CacheFull:
            for r in fresh:
                if r in state.live:
                    state.release(r)
            raise
        held = [state.live[r] for r in rids]
        batch = self._batch(rids, held, [len(p.tokens) for p in portions],
                            any(len(h.pages) != pages.get(r)
                                for r, h in zip(rids, held)))
        ids = [t for j in batch.order for t in portions[j].tokens]
        x = torch.tensor(ids, dtype=torch.long, device=self.device)
        start = {batch.order[e]: batch.host[e][0] for e in range(len(portions))}
        rows = torch.tensor([start[j] + int(w) for j, p in enumerate(portions)
                             for w in p.want], dtype=torch.long,
                            device=self.device)
        logits = self.model.run(x, batch, state, rows=rows)
        for p, h in zip(portions, held):
            h.length += len(p.tokens)
        return logits

    def _batch(self, rids, held, lens, grew: bool) -> RaggedBatch:
        """The batch's description; a step of single tokens by the same
        requests moves the previous one on, on the device."""
        key = tuple((r, h.slot, h.length) for r, h in zip(rids, held))
        if (not grew and self._last is not None and key == self._last_key
                and max(lens) == 1):
            batch = self._last
            batch.advance()
        else:
            batch = RaggedBatch(list(zip(held, lens)), self.device)
        single = max(lens) == 1
        self._last = batch if single else None
        self._last_key = tuple((r, h.slot, h.length + 1)
                               for r, h in zip(rids, held)) if single else None
        return batch

    def end(self, rid: Hashable):
        """The request is finished; its pages and slot are free again."""
        self.state.release(rid)


@dataclass
class Request:
    """One generation: a prompt, its sampling, and what came of it."""
    rid: Hashable
    prompt: List[int]
    params: SamplingParams
    max_tokens: int
    eos: frozenset = frozenset()
    done_prompt: int = 0
    output: List[int] = field(default_factory=list)
    finished: bool = False
    sampler: Optional[Sampler] = None

    @property
    def need(self) -> int:
        """Tokens it may come to hold (the last sampled one is never run)."""
        return len(self.prompt) + self.max_tokens - 1


class BatchScheduler:
    def __init__(self, engine: BatchEngine, token_budget: int = 2048):
        if token_budget < 1:
            raise ValueError("token_budget must be positive")
        self.engine = engine
        self.token_budget = token_budget
        self.waiting: Deque[Request] = deque()
        self.running: List[Request] = []
        self._reserved: Dict[Hashable, int] = {}
        self._next = 0

    @property
    def busy(self) -> bool:
        return bool(self.waiting or self.running)

    def submit(self, prompt: Sequence[int], params: Optional[SamplingParams] = None,
               max_tokens: int = 256, eos=()) -> Request:
        prompt = [int(t) for t in prompt]
        if not prompt:
            raise ValueError("empty prompt")
        if max_tokens < 1:
            raise ValueError("max_tokens must be positive")
        req = Request(self._next, prompt, params or SamplingParams(), max_tokens,
                      frozenset(int(e) for e in eos))
        if self._pages(req.need) > self.engine.state.n_pages:
            raise CacheFull(f"a request of {req.need} tokens does not fit the "
                            f"pool of {self.engine.state.n_pages * PAGE}")
        self._next += 1
        req.sampler = Sampler(req.params, prompt)
        self.waiting.append(req)
        return req

    def cancel(self, req: Request):
        """Stop a request wherever it is."""
        if req in self.waiting:
            self.waiting.remove(req)
        elif req in self.running:
            self._finish(req)
        req.finished = True

    @staticmethod
    def _pages(tokens: int) -> int:
        return (tokens + PAGE - 1) // PAGE

    def _finish(self, req: Request):
        req.finished = True
        self.running.remove(req)
        self._reserved.pop(req.rid)
        if req.rid in self.engine.state.live:
            self.engine.end(req.rid)

    def _admit(self):
        state = self.engine.state
        while self.waiting and len(self.running) < state.n_slots:
            need = self._pages(self.waiting[0].need)
            if sum(self._reserved.values()) + need > state.n_pages:
                return
            req = self.waiting.popleft()
            self._reserved[req.rid] = need
            self.running.append(req)

    def step(self) -> List[Tuple[Request, int, torch.Tensor]]:
        """One forward; returns (request, token, logprobs) of every request
        that got a token."""
        self._admit()
        budget = self.token_budget
        portions, sampled = [], []
        decoding = [r for r in self.running if r.done_prompt == len(r.prompt)]
        prompts = [r for r in self.running if r.done_prompt < len(r.prompt)]
        for r in decoding:
            portions.append(Portion(r.rid, [r.output[-1]], [0]))
            sampled.append(r)
            budget -= 1
        for r in prompts:
            if budget < 1:
                break
            part = r.prompt[r.done_prompt: r.done_prompt + budget]
            r.done_prompt += len(part)
            budget -= len(part)
            last = r.done_prompt == len(r.prompt)
            portions.append(Portion(r.rid, part, [len(part) - 1] if last else []))
            if last:
                sampled.append(r)
        if not portions:
            return []
        logits = self.engine.step(portions)
        out = []
        for r, (tok, logprobs) in zip(sampled, Sampler.draw_all(
                [r.sampler for r in sampled], logits)):
            r.output.append(tok)
            out.append((r, tok, logprobs))
            if tok in r.eos or len(r.output) >= r.max_tokens:
                self._finish(r)
        return out

    def generate(self, req: Request) -> Iterator[Tuple[int, torch.Tensor]]:
        """Step until one request is finished, yielding its tokens."""
        try:
            while not req.finished:
                for r, tok, logprobs in self.step():
                    if r is req:
                        yield tok, logprobs
        finally:
            if not req.finished:
                self.cancel(req)


class BatchService:
    """A scheduler on a thread of its own, fed by any number of callers.  Only
    that thread touches the scheduler; callers leave it notes."""

    def __init__(self, scheduler: BatchScheduler):
        self.scheduler = scheduler
        self._notes: queue.Queue = queue.Queue()
        self._streams: Dict[Hashable, queue.Queue] = {}
        self._requests: Dict[int, Request] = {}
        self._stopping = False
        self._thread = threading.Thread(target=self._loop, daemon=True)
        self._thread.start()

    # -- service thread ----------------------------------------------------
    def _loop(self):
        while not self._stopping:
            self._read_notes()
            if self._stopping or not self.scheduler.busy:
                continue
            try:
                events = self.scheduler.step()
            except Exception as e:  # noqa: BLE001 — every caller hears of it
                for r in [*self.scheduler.running, *self.scheduler.waiting]:
                    self.scheduler.cancel(r)
                self._fail(e)
                continue
            for r, tok, logprobs in events:
                out = self._streams.get(r.rid)
                if out is not None:
                    out.put((tok, logprobs))
                    if r.finished:
                        out.put(None)
        self._fail(RuntimeError("the service was stopped"))

    def _read_notes(self):
        block = not self.scheduler.busy
        while True:
            try:
                note = self._notes.get(block=block)
            except queue.Empty:
                return
            block = False
            if note is None:
                self._stopping = True
                return
            out, prompt, params = note
            if prompt is None:              # the caller went away
                req = self._requests.pop(id(out), None)
                if req is not None:
                    self._streams.pop(req.rid, None)
                    if not req.finished:
                        self.scheduler.cancel(req)
                continue
            try:
                req = self.scheduler.submit(prompt, params,
                                            params.max_tokens or 256)
            except Exception as e:  # noqa: BLE001 — reported to the caller
                out.put(e)
                continue
            self._streams[req.rid] = out
            self._requests[id(out)] = req

    def _fail(self, e: Exception):
        for out in self._streams.values():
            out.put(e)

    # -- callers -----------------------------------------------------------
    def generate(self, prompt: Sequence[int], params: SamplingParams
                 ) -> Generator[Tuple[int, torch.Tensor], None, None]:
        """Token stream of one request; closing it ends the request."""
        out: queue.Queue = queue.Queue()
        self._notes.put((out, list(prompt), params))
        try:
            while True:
                item = out.get()
                if item is None:
                    return
                if isinstance(item, Exception):
                    raise item
                yield item
        finally:
            self._notes.put((out, None, None))

    def stop(self):
        self._notes.put(None)
        self._thread.join()
