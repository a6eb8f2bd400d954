"""Prefill and decode throughput of layer stacks at real sizes (random weights).

Stacks of four layers of one kind with equal width, heads, key/value heads, head
sizes, latent size and feed-forward, so that their times compare directly:

  mla     DeepSeek-V2 latent attention + dense MLP (the closest existing model)
  latent  Tuvutar latent attention
  shared  Tuvutar latent attention, three of four layers on shared rows
  delta   Tuvutar gated delta rule
  mixed   Tuvutar delta, delta, delta, latent
  llama   Llama grouped attention + gated MLP (the closest model to the next)
  lepizen Lepizen grouped attention beside an ungated MLP of the same width
  moe     DeepSeek-V2 latent attention + routed experts (the closest model to
          the rest: equal experts, gated there and ungated here)
  windowed  Sadosun windowed attention + routed experts
  scan    Sadosun selective scan + routed experts
  sadosun Sadosun scan, windowed, windowed, scan
  gated   Dufinex attention + dense MLP (beside llama)
  reader  the same, three of four layers on another's keys and values
  channel Dufinex delta rule with decays per channel + dense MLP (beside delta)
  routed  Dufinex attention + routed experts (beside moe: equal experts)
  dufinex Dufinex delta, attention, attention on shared keys, delta + experts

All run the pipeline worker's own prefill and graph-captured decode step.
"""

from __future__ import annotations

import json
import time
from typing import Dict, Optional, Sequence

import torch

from ..config import ModelConfig
from ..parallel.rccl import PipelineWorker, build_stage_model
from .presets import (_dense_mla, _dufinex, _lepizen, _llama, _moe_mla,
                      _sadosun, _tuvutar)

SIZES: Dict[str, dict] = {
    "2048": dict(width=2048, heads=16, ff=8192, vocab=8192),
    "4096": dict(width=4096, heads=32, ff=14336, vocab=8192),
}
TUVUTAR = {"latent": "aaaa", "shared": "asss", "delta": "dddd", "mixed": "ddda"}
SADOSUN = {"windowed": "aaaa", "scan": "mmmm", "sadosun": "maam"}
DUFINEX = {"gated": "aaaa", "reader": "asss", "channel": "dddd",
           "routed": "AAAA", "dufinex": "dasD"}
EXPERT_FF = {"2048": 1408, "4096": 1536}
KINDS = ("mla", *TUVUTAR, "llama", "lepizen", "moe", *SADOSUN,
         *DUFINEX)
PREFILL = ((1, 8192), (8, 1024))     # sequences, tokens each
DECODE = ((1, 2048), (64, 2048))     # sequences, tokens cached


def stack(kind: str, size: dict) -> ModelConfig:
    if kind == "mla":
        return ModelConfig.from_dict(_dense_mla(n_layers=4, **size))
    if kind in ("llama", "lepizen"):
        make = _llama if kind == "llama" else _lepizen
        return ModelConfig.from_dict(
            make(n_layers=4, kv_heads=size["heads"] // 4, **size))
    if kind in DUFINEX:
        heads = size["heads"]
        return ModelConfig.from_dict(_dufinex(
            period=DUFINEX[kind], kv_heads=heads // 4, delta_heads=heads,
            delta_kv=heads // 2, expert_ff=EXPERT_FF[str(size["width"])], **size))
    if kind == "moe" or kind in SADOSUN:
        size = {**size, "ff": EXPERT_FF[str(size["width"])]}
        if kind == "moe":
            return ModelConfig.from_dict(_moe_mla(n_layers=4, **size))
        return ModelConfig.from_dict(
            _sadosun(period=SADOSUN[kind], kv_heads=size["heads"] // 4, **size))
    extra = {}
    if "d" in TUVUTAR[kind]:
        extra = dict(delta_heads=size["heads"], delta_kv=size["heads"] // 2)
    return ModelConfig.from_dict(
        _tuvutar(period=TUVUTAR[kind], repeats=1, **size, **extra))


def _spread(model):
    """Random router weights, not random biases of the choice, pick the experts;
    they see rows of an ordinary size."""
    for name, p in model.named_parameters():
        if name.endswith(".correction"):
            p.data.zero_()
        elif p.dim() <= 1 and ".norm" in name:
            p.data.fill_(1.0)


def _time(fn, n: int) -> float:
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(n):
        fn()
    torch.cuda.synchronize()
    return (time.perf_counter() - t0) / n


def run(which: str = "all", steps: int = 32,
        kinds: Optional[Sequence[str]] = None):
    if not torch.cuda.is_available():
        raise SystemExit("--layers needs a GPU")
    device = torch.device("cuda", 0)
    torch.manual_seed(0)
    for name in (SIZES if which == "all" else [which]):
        for kind in kinds or KINDS:
            config = stack(kind, SIZES[name])
            model = build_stage_model(config, 0, 1, device)
            if kind in SADOSUN or kind in DUFINEX:
                _spread(model)

            def emit(phase, batch, seq, seconds, tokens):
                print(json.dumps({
                    "metric": f"{phase} throughput, 4 layers", "kind": kind,
                    "width": int(name), "batch": batch, "seq_len": seq,
                    "ms": round(seconds * 1e3, 4),
                    "value": round(tokens / seconds, 1), "unit": "tokens/s",
                    "dtype": "bf16", "data": "synthetic"}), flush=True)

            for batch, seq in PREFILL:
                worker = PipelineWorker(model, 0, 1, device)
                ids = [torch.randint(0, config.vocab_size, (batch, seq),
                                     device=device)]
                fn = lambda: worker.prefill(ids, batch, 1, seq)  # noqa: E731
                fn(), fn()
                emit("prefill", batch, seq, _time(fn, 6), batch * seq)
            for batch, seq in DECODE:
                worker = PipelineWorker(model, 0, 1, device)
                ids = [torch.randint(0, config.vocab_size, (batch, seq),
                                     device=device)]
                tokens = worker.prefill(ids, batch, 1, seq)
                for _ in range(2):
                    tokens = worker.decode_step(tokens, batch, 1)
                if not worker.enable_graph_decode(tokens, batch, 1,
                                                  seq + steps + 16):
                    raise RuntimeError(f"{kind}: decode could not be captured")
                for _ in range(3):
                    tokens = worker.decode_step(tokens, batch, 1)
                emit("decode", batch, seq,
                     _time(lambda: worker.decode_step(tokens, batch, 1), steps),
                     batch)
                del worker
            del model
            torch.cuda.empty_cache()
