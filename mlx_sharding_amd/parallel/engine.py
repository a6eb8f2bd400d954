"""Driver-side generation loop over a chain of pipeline stages.

Mirrors the reference's driver loops (greedy CLI at
/root/reference/generate.py:52-88; full-sampling closure at
/root/reference/shard/utils.py:111-188): local first shard forward →
chain remote stages → sample on the last logits.  Remote stages are
abstract (`StageHandle`): gRPC clients (CPU plumbing / cross-node) or
the RCCL in-node pipeline (parallel/rccl.py).
"""

from __future__ import annotations

import time
from dataclasses import dataclass
from typing import Generator, Iterable, List, Optional, Protocol, Tuple

import torch

from .. import ops
from ..models.base import StageModel
from ..ops.kvcache import KVCache


class StageHandle(Protocol):
    def send_tensor(self, t: torch.Tensor, wire_fp16: bool = False,
                    device: str = "cpu") -> torch.Tensor: ...

    def reset_cache(self) -> None: ...


@dataclass
class SamplingParams:
    temperature: float = 0.0
    top_p: float = 1.0
    repetition_penalty: Optional[float] = None
    repetition_context_size: int = 20
    logit_bias: Optional[dict] = None
    seed: Optional[int] = None
    # upper bound on tokens this generation will draw (sizing hint for
    # graph-captured serving decode; the caller still enforces its own
    # stop conditions)
    max_tokens: Optional[int] = None


class Sampler:
    """Token choice of one generation: logit bias, repetition penalty over the
    recent context, temperature / top-p, with a generator of its own if seeded.
    """

    def __init__(self, params: SamplingParams, context: Iterable[int]):
        self.params = params
        self.context: List[int] = list(context)
        self.gen = None
        if params.seed is not None:
            self.gen = torch.Generator(device="cpu").manual_seed(params.seed)

    @property
    def plain(self) -> bool:
        """Greedy on the logits as they are."""
        p = self.params
        return (p.temperature <= 0.0 and not p.logit_bias
                and p.repetition_penalty in (None, 0, 1.0))

    def adjust(self, logits: torch.Tensor) -> torch.Tensor:
        """logits [1, V] with bias and penalty applied."""
        p, device = self.params, logits.device
        if p.logit_bias:
            idx = torch.tensor(list(p.logit_bias.keys()), device=device)
            vals = torch.tensor(list(p.logit_bias.values()), device=device,
                                dtype=logits.dtype)
            logits[0, idx] += vals
        if p.repetition_penalty and p.repetition_penalty != 1.0:
            window = self.context[-p.repetition_context_size:] \
                if p.repetition_context_size else self.context
            ctx = torch.tensor(window, device=device, dtype=torch.long)
            logits = ops.apply_repetition_penalty(logits, ctx,
                                                  p.repetition_penalty)
        return logits

    def sample(self, logits: torch.Tensor) -> torch.Tensor:
        """[1, V] adjusted logits -> [1] token, still on the device."""
        return ops.sample(logits, self.params.temperature, self.params.top_p,
                          self.gen)

    @staticmethod
    def draw_all(samplers: List["Sampler"], logits: torch.Tensor
                 ) -> List[Tuple[int, torch.Tensor]]:
        """One token per sampler from logits [n, V]; returns (token, logprobs).
        Plain greedy rows are chosen together."""
        if not samplers:
            return []
        if all(s.plain for s in samplers):
            toks = logits.argmax(-1).tolist()
        else:
            logits = logits.clone()
            toks = []
            for i, s in enumerate(samplers):
                row = s.adjust(logits[i: i + 1])
                logits[i] = row[0]
                # a seeded draw uses the host generator
                toks.append(int(s.sample(row.cpu() if s.gen is not None else row)))
        logprobs = torch.log_softmax(logits, -1)
        for s, t in zip(samplers, toks):
            s.context.append(t)
        return [(t, logprobs[i]) for i, t in enumerate(toks)]


def generate_step(
    prompt_ids: torch.Tensor,
    model: StageModel,
    cache: List[KVCache],
    remotes: Iterable[StageHandle] = (),
    params: Optional[SamplingParams] = None,
    wire_fp16: bool = False,
    prefill_chunk: int = 0,
    prefill_from: int = 0,
) -> Generator[Tuple[int, torch.Tensor], None, None]:
    """Yield (token_id, logprobs[V]) forever; caller decides when to stop.

    Resets every remote stage's cache at generator start (the
    reference's per-request lifecycle, utils.py:122-124); the local
    ``cache`` must be fresh.

    ``prefill_chunk`` > 0 feeds the prompt in chunks of that many
    tokens (bounded activation memory for long prompts; each chunk is
    one more SendTensor to the remote stages, whose caches accumulate
    — the on-GPU chunked-prefill equivalence is kernel-tested).

    ``prefill_from`` > 0 skips prefilling the first N prompt tokens:
    the caller guarantees ``cache`` already holds their K/V (prefix
    caching — the caches were trimmed to exactly N).  Only valid
    without remotes (remote stages have no trim control channel);
    0 < prefill_from < prompt length.
    """
    params = params or SamplingParams()
    remotes = list(remotes)
    if prefill_from:
        if remotes:
            raise ValueError("prefill_from requires a purely local chain")
        if not 0 < prefill_from < prompt_ids.shape[1]:
            raise ValueError(f"prefill_from {prefill_from} outside "
                             f"(0, {prompt_ids.shape[1]})")
        if any(c.offset != prefill_from for c in cache):
            raise ValueError("cache offsets do not match prefill_from")
    for r in remotes:
        r.reset_cache()
    device = prompt_ids.device
    sampler = Sampler(params, prompt_ids[0].tolist())

    def _forward(y):
        h = model(y, cache)
        for r in remotes:
            h = r.send_tensor(h, wire_fp16=wire_fp16, device=str(device))
        return h

    with torch.no_grad():
        fresh = prompt_ids[:, prefill_from:] if prefill_from else prompt_ids
        if prefill_chunk and fresh.shape[1] > prefill_chunk:
            for c0 in range(0, fresh.shape[1], prefill_chunk):
                h = _forward(fresh[:, c0: c0 + prefill_chunk])
        else:
            h = _forward(fresh)
        while True:
            logits = sampler.adjust(h[:, -1, :].float())
            logprobs = logits - torch.logsumexp(logits, dim=-1, keepdim=True)
            tok = sampler.sample(logits)
            # one-step lookahead (the reference's mx.async_eval,
            # generate.py:82-88): enqueue the NEXT forward before the
            # host sync on .item(), hiding its launch latency behind
            # the caller's per-token work.  The final lookahead step is
            # wasted compute, exactly as in the reference.
            h = _forward(tok.reshape(-1, 1))
            tid = int(tok.item())
            sampler.context.append(tid)
            yield tid, logprobs[0]


def batched_generate_step(prompt_ids: torch.Tensor, model: StageModel,
                          params: Optional[SamplingParams], max_tokens: int,
                          prefill_chunk: int = 0
                          ) -> Generator[Tuple[int, torch.Tensor], None, None]:
    """generate_step for a model that runs ragged batches: one request through
    the batch scheduler, ending by itself after ``max_tokens``."""
    from .batching import PAGE, BatchEngine, BatchScheduler
    need = prompt_ids.shape[1] + max_tokens
    engine = BatchEngine(model, (need + PAGE - 1) // PAGE * PAGE, 1)
    sched = BatchScheduler(engine, prefill_chunk or 2048)
    return sched.generate(sched.submit(prompt_ids[0].tolist(), params, max_tokens))


@dataclass
class GenerationStats:
    prompt_tokens: int = 0
    generation_tokens: int = 0
    prompt_tps: float = 0.0
    generation_tps: float = 0.0
    ttft_s: float = 0.0


def stream_generate(
    prompt_ids: torch.Tensor,
    model: StageModel,
    remotes: Iterable[StageHandle] = (),
    max_tokens: int = 256,
    params: Optional[SamplingParams] = None,
    eos_token_ids: Iterable[int] = (),
    wire_fp16: bool = False,
    stats: Optional[GenerationStats] = None,
) -> Generator[Tuple[int, torch.Tensor], None, None]:
    """Token stream with EOS stop + the reference's TPS accounting
    (prompt TPS = prompt_tokens / time-to-first-token; gen TPS =
    (n-1)/decode_time — /root/reference/generate.py:103-122)."""
    eos = set(int(e) for e in eos_token_ids)
    remotes = list(remotes)
    t0 = time.perf_counter()
    n = 0
    t_first = t0
    if model.supports_ragged and not remotes and prompt_ids.shape[0] == 1:
        tokens = batched_generate_step(prompt_ids, model, params, max_tokens)
    else:
        tokens = generate_step(prompt_ids, model,
                               model.make_cache(batch_size=prompt_ids.shape[0]),
                               remotes, params, wire_fp16)
    for tid, logprobs in tokens:
        if n == 0:
            t_first = time.perf_counter()
        n += 1
        if tid in eos:
            break
        yield tid, logprobs
        if n >= max_tokens:
            break
    t_end = time.perf_counter()
    if stats is not None:
        stats.prompt_tokens = int(prompt_ids.shape[1])
        stats.generation_tokens = n
        stats.ttft_s = t_first - t0
        stats.prompt_tps = stats.prompt_tokens / max(t_first - t0, 1e-9)
        stats.generation_tps = (n - 1) / max(t_end - t_first, 1e-9) if n > 1 else 0.0


class LocalChain:
    """In-process stage chain (testing + PP=1): behaves like a remote."""

    def __init__(self, model: StageModel, batch_size: int = 1):
        self.model = model
        self.batch_size = batch_size
        self.cache = None

    def send_tensor(self, t: torch.Tensor, wire_fp16: bool = False,
                    device: str = "cpu") -> torch.Tensor:
        if wire_fp16 and t.dtype == torch.bfloat16:
            t = t.to(torch.float16)
        x = t.to(self.model.hop_dtype) if t.is_floating_point() else t
        if self.cache is None or (self.cache and self.cache[0].batch_size != x.shape[0]):
            self.cache = self.model.make_cache(batch_size=x.shape[0])
        with torch.no_grad():
            return self.model(x, self.cache)

    def reset_cache(self):
        self.cache = None
