"""What the designs that run ragged batches have in common.

config.json gives ``width``, ``vocab``, ``norm.eps`` and ``layers``, a list of
{"type", "mixer", "mlp"}.  Tensors: ``embed``, ``l<i>.*``, ``final.norm``,
``head`` (where it is not the embedding table).  The residual stream is 32-bit,
also between pipeline stages.  A layer whose mixer has ``kv_from`` reads the rows
that layer cached, so both live on one stage.
"""

from __future__ import annotations

import re
from typing import Dict, List, Optional, Tuple

import torch
import torch.nn as nn
import torch.nn.functional as F

from .. import ops
from ..config import ModelConfig, ShardSpec
from ..ops.paged import PagedState, RaggedBatch, RaggedCache, RaggedLayerCache
from ..ops.ragged import Rotary
from .base import Linear, RMSNorm, StageModel, owned_layer_indices


class RaggedStageModel(StageModel):
    """A stage of a design with layers ``l<i>`` over a PagedState.  A design
    makes its layer modules (``make_layer``; each has a ``mix`` with a
    ``store_spec``) and the forward over a batch (``run``)."""

    supports_ragged = True
    supports_quantization = False
    norm_offset = 0.0  # norm weights are stored around 1 - norm_offset
    tied_head = False  # the embedding table makes the logits
    # parameters that are not the ``weight`` of a module
    bare_parameters: Tuple[str, ...] = ()

    def __init__(self, config: ModelConfig, shard: ShardSpec, quant_for=None,
                 dtype: torch.dtype = torch.bfloat16):
        super().__init__(config, shard)
        W, self.eps = config.hidden_size, float(config["norm"]["eps"])
        if shard.is_first or (self.tied_head and shard.is_last):
            self.embed = nn.Embedding(config.vocab_size, W, dtype=dtype)
        for i in owned_layer_indices(shard):
            self.add_module(f"l{i}", self.make_layer(i, config["layers"][i],
                                                     W, dtype))
        if shard.is_last:
            self.final = nn.Module()
            self.final.norm = self.make_final_norm(W, dtype)
            if not self.tied_head:
                self.head = Linear(W, config.vocab_size, dtype=dtype)
        self._tables: Dict = {}
        self._old_tables: List = []  # captured graphs may still read them
        for i in owned_layer_indices(shard):
            j = config["layers"][i]["mixer"].get("kv_from")
            if j is not None and not (shard.owns(int(j)) and int(j) < i):
                raise ValueError(
                    f"layer {i} reads the rows of layer {j}, which stage "
                    f"[{shard.start_layer}, {shard.end_layer}) does not run "
                    f"before it")

    def make_layer(self, i: int, spec: dict, width: int,
                   dtype: torch.dtype) -> nn.Module:
        raise NotImplementedError

    def make_final_norm(self, width: int, dtype: torch.dtype) -> nn.Module:
        return RMSNorm(width, self.eps, self.norm_offset, dtype)

    # -- layers that read another layer's rows -----------------------------
    @staticmethod
    def row_source(config: ModelConfig, i: int) -> int:
        """The layer whose rows layer i reads."""
        j = config["layers"][i]["mixer"].get("kv_from")
        return i if j is None else int(j)

    @classmethod
    def allowed_cuts(cls, config: ModelConfig) -> Optional[List[int]]:
        """Layer indices a pipeline stage may begin at: not between a layer
        and one that reads its rows (None: any)."""
        n = config.num_hidden_layers
        bad = set()
        for i in range(n):
            bad.update(range(cls.row_source(config, i) + 1, i + 1))
        return [c for c in range(1, n) if c not in bad] if bad else None

    def layer(self, i: int) -> nn.Module:
        return getattr(self, f"l{i}")

    def layer_items(self):
        return [(i, self.layer(i)) for i in owned_layer_indices(self.shard)]

    @property
    def hop_dtype(self) -> torch.dtype:
        return torch.float32  # stages hand on the residual stream

    # -- weights -----------------------------------------------------------
    @classmethod
    def owns_key(cls, key: str, shard: ShardSpec) -> bool:
        top = key.split(".")[0]
        if top == "embed":
            return shard.is_first or (cls.tied_head and shard.is_last)
        if top in ("final", "head"):
            return shard.is_last
        return top[:1] == "l" and top[1:].isdigit() and shard.owns(int(top[1:]))

    @classmethod
    def sanitize(cls, weights, shard: ShardSpec):
        out = {}
        for k, v in cls.stack_experts(weights, shard).items():
            if cls.owns_key(k, shard):
                if k.rsplit(".", 1)[-1] not in (*cls.bare_parameters, "weight"):
                    k = f"{k}.weight"
                out[k] = v
        return out

    @classmethod
    def stack_experts(cls, weights, shard: ShardSpec):
        """One stacked matrix per kind in place of those of the experts."""
        found: Dict[str, Dict[int, str]] = {}
        out = dict(weights)
        for k in weights:
            m = re.fullmatch(r"(l\d+\.mlp)\.e(\d+)\.(gate|up|down)", k)
            if m and cls.owns_key(k, shard):
                found.setdefault(f"{m[1]}.{m[3]}", {})[int(m[2])] = k
        for name, keys in found.items():
            if sorted(keys) == list(range(len(keys))):  # else: reported
                out[name] = torch.stack([out.pop(keys[e])
                                         for e in range(len(keys))])
        return out

    # -- cache -------------------------------------------------------------
    def store_specs(self) -> List:
        return [self.layer_spec(layer) for _, layer in self.layer_items()]

    def layer_spec(self, layer: nn.Module):
        """What one layer keeps between steps (ops.paged)."""
        return layer.mix.store_spec()

    def make_state(self, max_tokens: int, max_requests: int) -> PagedState:
        p = next(self.parameters())
        return PagedState(self.store_specs(), max_tokens, max_requests,
                          p.dtype, p.device)

    def make_cache(self, dtype: Optional[torch.dtype] = None,
                   batch_size: int = 1, device=None) -> List[RaggedLayerCache]:
        p = next(self.parameters())
        shared = RaggedCache(self.store_specs(), batch_size, dtype or p.dtype,
                             device if device is not None else p.device)
        return [RaggedLayerCache(shared, i) for i in range(self.shard.n_layers)]

    # -- forward -----------------------------------------------------------
    def _rotation(self, rotary: Rotary, n: int, device):
        """(cos, sin) tables of at least n positions."""
        got = self._tables.get(rotary)
        if got is None or got[0].shape[0] < n or got[0].device != device:
            if got is not None:
                self._old_tables.append(got)
            rows = max(1024, 1 << max(n - 1, 1).bit_length())
            got = self._tables[rotary] = rotary.tables(rows, device)
        return got

    def residual(self, x: torch.Tensor) -> torch.Tensor:
        """What the first owned layer adds to: embedded token ids, or a copy
        of the residual stream that the previous stage handed on."""
        if self.shard.is_first:
            return F.embedding(x, self.embed.weight).float()
        return x[:, : self.config.hidden_size].float().contiguous().clone()

    def logits(self, h: torch.Tensor) -> torch.Tensor:
        """fp32 logits of rows that went through the final norm."""
        if self.tied_head:
            return ops.linear(h, self.embed.weight).float()
        return self.head(h).float()

    def run(self, x: torch.Tensor, batch: RaggedBatch, state: PagedState,
            rows: Optional[torch.Tensor] = None,
            layer_outputs: Optional[list] = None) -> torch.Tensor:
        """One ragged forward.  x: token ids [N] on the first stage, else what
        the previous stage returned; rows select the tokens that go through
        the head.  Returns what the next stage takes, or fp32 logits."""
        raise NotImplementedError

    def forward(self, x: torch.Tensor, cache: Optional[List] = None) -> torch.Tensor:
        B, T = x.shape[:2]
        if cache is None:
            cache = self.make_cache(batch_size=B, device=x.device)
        shared = cache[0].shared
        if B != shared.batch_size:
            raise ValueError(f"cache batch mismatch: {shared.batch_size} vs {B}")
        y = self.run(x.reshape(B * T, *x.shape[2:]), shared.next_batch(T),
                     shared.state)
        return y.view(B, T, -1)
