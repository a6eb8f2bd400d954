"""Dufinex stage model: grouped attention and a delta rule with a decay per
channel in any order, dense or routed feed-forwards.

config.json: ``width``, ``vocab``, ``norm.eps``, ``embedding.scale`` and
``layers``, a list of {"type", "mixer", "mlp"}.  A sublayer reads the 32-bit
residual stream as it is, and its output is normed before it is added; ``mlp``
may be null.  Attention has no positions; a layer with ``kv_from`` reads the keys
and values that layer cached.  The ranks of a delta layer's decay and gate are
``decay_rank`` and ``gate_rank`` of its mixer, or those of its tensors.

Tensors: ``embed`` (the head, too), ``l<i>.norm1`` / ``norm2``, ``l<i>.mix.*``,
``l<i>.mlp.*`` (``.b``: a projection's bias; ``.e<j>.*``: an expert's), ``final.norm``.
"""

from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from ..config import ModelConfig
from ..ops import ragged
from ..ops.experts import ExpertShape, Routing
from ..ops.paged import PagedState, RaggedBatch
from ..ops.ragged import ClampedGLU
from .base import RMSNorm
from .mixers import BiasedMLP, GatedDelta, GroupedAttention, RoutedExperts
from .ragged import RaggedStageModel

ROUTING = Routing(score="sigmoid", normalize=False, on_input=True)


def _mixer(kind: str, mx: dict, width: int, eps: float, dtype: torch.dtype):
    heads, kv_heads = int(mx["heads"]), int(mx["kv_heads"])
    dim, vdim = int(mx["dim"]), int(mx["vdim"])
    if kind == "attention":
        return GroupedAttention(
            width, heads, kv_heads, dim, vdim, float(mx["scale"]), eps,
            sink=True, dtype=dtype, head_weights=True, gate=True,
            own_rows=mx.get("kv_from") is None)
    if kind == "channel_delta":
        return GatedDelta(
            width, heads, kv_heads, dim, vdim, int(mx["conv"]), eps, dtype,
            ranks=(int(mx["decay_rank"]), int(mx["gate_rank"])), gate="sigmoid")
    raise ValueError(f"unknown mixer type {kind!r}")


def _mlp(spec: dict, width: int, dtype: torch.dtype):
    if spec["kind"] == "dense":
        return BiasedMLP(width, int(spec["ff"]),
                         ClampedGLU(float(spec["limit"])), dtype)
    if spec["kind"] == "moe":
        expert, router = spec["expert"], spec["router"]
        return RoutedExperts(
            width, int(expert["ff"]), int(router["experts"]), 0,
            int(router["top"]), dtype, glu=ClampedGLU(float(expert["limit"])),
            routing=ROUTING, correction=False)
    raise ValueError(f"unknown feed-forward kind {spec['kind']!r}")


class DufinexLayer(nn.Module):
    def __init__(self, spec: dict, width: int, eps: float, dtype: torch.dtype):
        super().__init__()
        self.mix = _mixer(spec["type"], spec["mixer"], width, eps, dtype)
        self.norm1 = RMSNorm(width, eps, dtype=dtype)
        self.mlp = None
        if spec.get("mlp") is not None:
            self.mlp = _mlp(spec["mlp"], width, dtype)
            self.norm2 = RMSNorm(width, eps, dtype=dtype)


class DufinexStageModel(RaggedStageModel):
    model_type = "dufinex"
    bare_parameters = ("A_log", "dt_bias", "sink", "bias")
    tied_head = True

    def __init__(self, config, shard, quant_for=None, dtype=torch.bfloat16):
        super().__init__(config, shard, quant_for, dtype)
        for i, layer in self.layer_items():
            src = self.row_source(config, i)
            if src == i:
                continue
            source = self.layer(src).mix
            if (not isinstance(source, GroupedAttention) or source.k is None
                    or source.shape != layer.mix.shape):
                raise ValueError(f"layer {i} cannot read the keys and values "
                                 f"of layer {src}")

    def make_layer(self, i, spec, width, dtype):
        return DufinexLayer(spec, width, self.eps, dtype)

    # -- weights -----------------------------------------------------------
    @classmethod
    def complete_config(cls, config: ModelConfig, weights):
        for i, spec in enumerate(config["layers"]):
            if spec["type"] != "channel_delta":
                continue
            for name, leaf in (("decay_rank", "a1"), ("gate_rank", "g1")):
                w = weights.get(f"l{i}.mix.{leaf}")
                if w is not None:
                    spec["mixer"].setdefault(name, w.shape[0])

    @classmethod
    def sanitize(cls, weights, shard):
        # a feed-forward's ".b" is a bias, a mixer's a projection
        return super().sanitize(
            {f"{k[:-1]}bias" if ".mlp." in k and k.endswith(".b") else k: v
             for k, v in weights.items()}, shard)

    # -- forward -----------------------------------------------------------
    @torch.no_grad()
    def run(self, x: torch.Tensor, batch: RaggedBatch, state: PagedState,
            rows: Optional[torch.Tensor] = None,
            layer_outputs: Optional[list] = None) -> torch.Tensor:
        W = self.config.hidden_size
        dtype = next(self.parameters()).dtype
        x = self.residual(x)
        if self.shard.is_first:
            x.mul_(float(self.config["embedding"]["scale"]))
        items = self.layer_items()
        first = self.shard.start_layer

        def add(y, norm, after=None, **of_y):
            """The residual moves on; returns what the next sublayer reads, or
            the rows of the norm that follows."""
            return ragged.add_norm(
                x, y, None if norm is None else norm.weight,
                None if after is None else after.weight, self.eps, 0.0, dtype,
                copy=True, pad_to=1 if after is not None else ExpertShape.STEP,
                **of_y)

        h = add(None, None)
        for k, (i, layer) in enumerate(items):
            store = state.layers[self.row_source(self.config, i) - first]
            last = k + 1 == len(items) and self.shard.is_last
            end = self.final.norm if last else None
            y = layer.mix(h[:, :W], batch, store)
            if isinstance(layer.mix, GroupedAttention):
                y = y[0]
            if layer.mlp is None:
                h = add(y, layer.norm1, end)
            else:
                h = add(y, layer.norm1)
                if isinstance(layer.mlp, RoutedExperts):
                    y, where = layer.mlp.rows(h)
                    h = add(y, layer.norm2, end, where=where)
                else:
                    y, bias = layer.mlp.rows(h[:, :W])
                    h = add(y, layer.norm2, end, y_bias=bias)
            if layer_outputs is not None:
                layer_outputs.append(x.clone())
        if not self.shard.is_last:
            return x
        if rows is not None:
            h = h.index_select(0, rows)
        return self.logits(h)
