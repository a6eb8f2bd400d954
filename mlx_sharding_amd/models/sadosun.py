"""Sadosun stage model: windowed attention and selective-scan layers in any
order, routed experts, and a token's own embedding row in every layer.

config.json: ``width``, ``vocab``, ``norm.eps``, ``embedding.scale``,
``canon.taps``, ``token_side.dim`` and ``layers``, a list of {"type", "mixer",
"mlp"}.  On a 32-bit residual stream, each sublayer reads its normed input (one
number as norm weight) plus a short causal convolution of it; ``mlp`` (routed
experts) may be null.  After both, every layer adds a gated projection of its
slice of the token's row in a second embedding table.  Those rows are known to
the first stage only, so the slices of later layers travel with the residual
stream.

Tensors: ``embed``, ``side.embed``, ``l<i>.norm1`` / ``norm2``, ``l<i>.canon1`` /
``canon2``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``l<i>.side.*``, ``final.norm``,
``head``.
"""

from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from ..config import ModelConfig, ShardSpec
from ..ops import ragged
from ..ops.experts import FEW, ExpertShape
from ..ops.paged import LayerSpec, PagedState, RaggedBatch
from ..ops.ragged import Rotary, Turns
from ..ops.recurrent import norm_conv
from .mixers import (CausalConv, GroupedAttention, RoutedExperts, ScalarNorm,
                     SelectiveScan, TokenInput)
from .ragged import RaggedStageModel


def _mixer(kind: str, mx: dict, width: int, eps: float, dtype: torch.dtype):
    if kind == "attention":
        base, vdim = float(mx["rot"]["base"]), int(mx["vdim"])
        return GroupedAttention(
            width, int(mx["heads"]), int(mx["kv_heads"]), int(mx["dim"]), vdim,
            float(mx["scale"]), eps, dtype=dtype, head_norm=True,
            rotary=Rotary(int(mx["rot"]["dims"]), base),
            turn_values=Rotary(vdim, base), window=int(mx["mask"]["size"]),
            zero_sink=True)
    if kind == "mamba1":
        return SelectiveScan(width, int(mx["inner"]), int(mx["state"]),
                             int(mx["dt_rank"]), int(mx["conv"]), dtype)
    raise ValueError(f"unknown mixer type {kind!r}")


class SadosunLayer(nn.Module):
    def __init__(self, spec: dict, width: int, eps: float, taps: int,
                 side: int, dtype: torch.dtype):
        super().__init__()
        self.norm1 = ScalarNorm(dtype)
        self.canon1 = CausalConv(width, taps, False, dtype)
        self.mix = _mixer(spec["type"], spec["mixer"], width, eps, dtype)
        mlp = spec.get("mlp")
        self.mlp = None
        if mlp is not None:
            if mlp["kind"] != "moe":
                raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
            r = mlp["router"]
            self.norm2 = ScalarNorm(dtype)
            self.canon2 = CausalConv(width, taps, False, dtype)
            self.mlp = RoutedExperts(
                width, int(mlp["expert"]["ff"]), int(r["experts"]),
                int(r.get("identity") or 0), int(r["top"]), dtype)
        self.side = TokenInput(width, side, eps, dtype)


class SadosunStageModel(RaggedStageModel):
    model_type = "sadosun"
    bare_parameters = ("A_log", "D", "b", "correction")

    def __init__(self, config: ModelConfig, shard: ShardSpec, quant_for=None,
                 dtype: torch.dtype = torch.bfloat16):
        super().__init__(config, shard, quant_for, dtype)
        if shard.is_first:
            self.side = nn.Module()
            self.side.embed = nn.Embedding(
                config.vocab_size, self.side_dim * config.num_hidden_layers,
                dtype=dtype)

    @property
    def side_dim(self) -> int:
        return int(self.config["token_side"]["dim"])

    @property
    def hop_width(self) -> int:
        left = self.config.num_hidden_layers - self.shard.start_layer
        return self.config.hidden_size + left * self.side_dim

    def make_layer(self, i, spec, width, dtype):
        return SadosunLayer(spec, width, self.eps,
                            int(self.config["canon"]["taps"]), self.side_dim,
                            dtype)

    def make_final_norm(self, width, dtype):
        return ScalarNorm(dtype)

    def layer_spec(self, layer):
        spec = layer.mix.store_spec()
        if not isinstance(spec, LayerSpec):
            spec = LayerSpec(spec, {})
        canon = {"canon1": layer.canon1.history()}
        if layer.mlp is not None:
            canon["canon2"] = layer.canon2.history()
        return LayerSpec(spec.mix, {**spec.histories, **canon})

    # -- weights -----------------------------------------------------------
    @classmethod
    def owns_key(cls, key, shard):
        if key.split(".")[0] == "side":
            return shard.is_first
        return super().owns_key(key, shard)

    # -- forward -----------------------------------------------------------
    def _turns(self, layer, batch: RaggedBatch, device) -> Turns:
        n = batch.max_pos
        return Turns(self._rotation(layer.mix.rotary, n, device),
                     self._rotation(layer.mix.turn_values, n, device))

    @torch.no_grad()
    def run(self, x: torch.Tensor, batch: RaggedBatch, state: PagedState,
            rows: Optional[torch.Tensor] = None,
            layer_outputs: Optional[list] = None) -> torch.Tensor:
        W, n = self.config.hidden_size, self.side_dim
        dtype = next(self.parameters()).dtype
        if self.shard.is_first:
            side = F.embedding(x, self.side.embed.weight)
            x = self.residual(x).mul_(float(self.config["embedding"]["scale"]))
        else:
            side = x[:, W:].to(dtype)
            x = self.residual(x)
        items = self.layer_items()

        def enter(k, which, y=None, post=None, pad_to=1):
            layer, store = items[k][1], state.layers[k]
            norm = getattr(layer, f"norm{which}")
            conv = getattr(layer, f"canon{which}")
            return norm_conv(x, y, post, norm.weight, self.eps, conv.by_tap,
                             store.histories[f"canon{which}"], batch, dtype,
                             pad_to)

        h = enter(0, 1)
        for k, (i, layer) in enumerate(items):
            if isinstance(layer.mix, GroupedAttention):
                y, _ = layer.mix(h, batch, state.layers[k], None,
                                 self._turns(layer, batch, x.device))
            else:
                y = layer.mix(h, batch, state.layers[k])
            copy = None
            if layer.mlp is not None:
                h = enter(k, 2, y, pad_to=ExpertShape.STEP)
                copy = layer.mlp(x, h, copy=batch.n_tokens > FEW)
            else:
                ragged.add_norm(x, y, None, None, self.eps, 0.0, dtype)
            at = k * n
            y = layer.side(x, side[:, at: at + n], copy)
            post = layer.side.norm.weight
            if k + 1 < len(items):
                h = enter(k + 1, 1, y, post)
            else:
                last = self.final.norm.weight if self.shard.is_last else None
                h = ragged.add_norm(x, y, post, last, self.eps, 0.0, dtype)
            if layer_outputs is not None:
                layer_outputs.append(x.clone())
        if not self.shard.is_last:
            return torch.cat([x, side[:, len(items) * n:].float()], 1)
        if rows is not None:
            h = h.index_select(0, rows)
        return self.logits(h)
