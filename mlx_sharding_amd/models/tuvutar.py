"""Tuvutar stage model: gated-delta and latent-attention layers in any order.

config.json: ``width``, ``vocab``, ``norm.eps`` and ``layers``, a list of
{"type", "mixer", "mlp"}.  A layer is normed on both sides of each sublayer
(norm weights stored around zero) on a 32-bit residual stream; ``mlp`` may be
null.  A latent-attention layer with ``kv_from`` reads the rows that layer
cached, so both live on the same pipeline stage.

Tensors: ``embed``, ``l<i>.norm1`` / ``norm1b`` / ``norm2`` / ``norm2b``,
``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``, ``head``.
"""

from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from ..ops import ragged
from ..ops.paged import PagedState, RaggedBatch
from ..ops.ragged import Rotary
from .base import RMSNorm
from .mixers import GatedDelta, GatedMLP, LatentAttention
from .ragged import RaggedStageModel

NORM_OFFSET = 1.0  # norm weights are stored around zero


def _rotary(rot: dict) -> Rotary:
    sc = rot.get("scaling")
    if not sc:
        return Rotary(int(rot["dims"]), float(rot["base"]))
    return Rotary(int(rot["dims"]), float(rot["base"]), float(sc["factor"]),
                  float(sc["original"]), float(sc["fast"]), float(sc["slow"]))


def _mixer(kind: str, mx: dict, width: int, eps: float, dtype: torch.dtype):
    if kind == "latent_attention":
        rotary = _rotary(mx["rot"])
        if rotary.dims != int(mx["rot_dim"]):
            raise ValueError("the rotated part has rot_dim = rot.dims dimensions")
        return LatentAttention(
            width, int(mx["heads"]), int(mx["dim"]), int(mx["vdim"]),
            int(mx["kv_rank"]), rotary, float(mx["scale"]), eps,
            own_rows=mx.get("kv_from") is None, dtype=dtype)
    if kind == "delta":
        return GatedDelta(width, int(mx["heads"]), int(mx["kv_heads"]),
                          int(mx["dim"]), int(mx["vdim"]), int(mx["conv"]),
                          eps, dtype=dtype)
    raise ValueError(f"unknown mixer type {kind!r}")


class TuvutarLayer(nn.Module):
    def __init__(self, spec: dict, width: int, eps: float, dtype: torch.dtype):
        super().__init__()
        mx = spec["mixer"]
        self.norm1 = RMSNorm(width, eps, NORM_OFFSET, dtype)
        self.norm1b = RMSNorm(width, eps, NORM_OFFSET, dtype)
        self.mix = _mixer(spec["type"], mx, width, eps, dtype)
        mlp = spec.get("mlp")
        self.mlp = None
        if mlp is not None:
            if mlp["kind"] != "dense":
                raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
            self.norm2 = RMSNorm(width, eps, NORM_OFFSET, dtype)
            self.norm2b = RMSNorm(width, eps, NORM_OFFSET, dtype)
            self.mlp = GatedMLP(width, int(mlp["ff"]), "gelu_tanh", dtype)


class TuvutarStageModel(RaggedStageModel):
    model_type = "tuvutar"
    norm_offset = NORM_OFFSET
    bare_parameters = ("A_log", "dt_bias")

    def make_layer(self, i, spec, width, dtype):
        return TuvutarLayer(spec, width, self.eps, dtype)

    # -- forward -----------------------------------------------------------
    @torch.no_grad()
    def run(self, x: torch.Tensor, batch: RaggedBatch, state: PagedState,
            rows: Optional[torch.Tensor] = None,
            layer_outputs: Optional[list] = None) -> torch.Tensor:
        x = self.residual(x)
        dtype = next(self.parameters()).dtype
        norm = lambda y, post, nxt: ragged.add_norm(  # noqa: E731
            x, y, None if post is None else post.weight,
            None if nxt is None else nxt.weight, self.eps, NORM_OFFSET, dtype)
        items = self.layer_items()
        first = self.shard.start_layer
        h = norm(None, None, items[0][1].norm1)
        for k, (i, layer) in enumerate(items):
            if k + 1 < len(items):
                after = items[k + 1][1].norm1
            else:
                after = self.final.norm if self.shard.is_last else None
            if isinstance(layer.mix, LatentAttention):
                src = self.row_source(self.config, i)
                y = layer.mix(h, batch, state.layers[src - first],
                              self._rotation(layer.mix.rotary, batch.max_pos,
                                             x.device))
            else:
                y = layer.mix(h, batch, state.layers[k])
            if layer.mlp is None:
                h = norm(y, layer.norm1b, after)
            else:
                h = norm(y, layer.norm1b, layer.norm2)
                h = norm(layer.mlp(h), layer.norm2b, after)
            if layer_outputs is not None:
                layer_outputs.append(x.clone())
        if not self.shard.is_last:
            return x
        if rows is not None:
            h = h.index_select(0, rows)
        return self.logits(h)
