"""Lepizen stage model: parallel layers of grouped softmax attention and an
ungated feed-forward.

config.json: ``width``, ``vocab``, ``norm.eps``, ``residual_mult``,
``logit_scale``, ``logit_softcap`` and ``layers``, a list of {"type", "mixer",
"mlp"}.  A layer norms the 32-bit residual stream once, both sublayers read
that, and ``residual_mult`` times their sum is added back; ``mlp`` may be null.
Attention has no positions, norms its whole query and key projections, and adds
a learned sink per head to the softmax.  Layers with ``v_mix`` blend the values
of the first such layer into their own, so those values travel with the
residual stream from stage to stage.

Tensors: ``embed``, ``l<i>.norm1``, ``l<i>.mix.*``, ``l<i>.mlp.*``,
``final.norm``, ``head``.
"""

from __future__ import annotations

from typing import Optional

import torch

from ..config import ModelConfig
from ..ops import ragged
from ..ops.paged import PagedState, RaggedBatch
from .base import RMSNorm
from .mixers import MLP, GroupedAttention, ParallelBlock
from .ragged import RaggedStageModel


class LepizenLayer(ParallelBlock):
    def __init__(self, spec: dict, width: int, eps: float, first_mix: bool,
                 dtype: torch.dtype):
        if spec["type"] != "attention":
            raise ValueError(f"unknown mixer type {spec['type']!r}")
        mx, mlp = spec["mixer"], spec.get("mlp")
        if mlp is not None and mlp["kind"] != "dense":
            raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
        super().__init__(
            GroupedAttention(width, int(mx["heads"]), int(mx["kv_heads"]),
                             int(mx["dim"]), int(mx["vdim"]),
                             float(mx["scale"]), eps, qk_norm=True, sink=True,
                             dtype=dtype),
            None if mlp is None else MLP(width, int(mlp["ff"]), "gelu", dtype))
        self.norm1 = RMSNorm(width, eps, dtype=dtype)
        self.mixes = bool(mx.get("v_mix")) and not first_mix


class LepizenStageModel(RaggedStageModel):
    model_type = "lepizen"
    bare_parameters = ("sink", "vmix")

    def make_layer(self, i, spec, width, dtype):
        return LepizenLayer(spec, width, self.eps,
                            i == self.first_mix(self.config), dtype)

    # -- values of the first mixing layer ----------------------------------
    @staticmethod
    def first_mix(config: ModelConfig) -> Optional[int]:
        for i, spec in enumerate(config["layers"]):
            if spec["mixer"].get("v_mix"):
                return i
        return None

    @classmethod
    def carried(cls, config: ModelConfig, cut: int) -> int:
        """Width of the values that a stage beginning at layer ``cut`` needs
        from before it."""
        j = cls.first_mix(config)
        if j is None or j >= cut or not any(
                s["mixer"].get("v_mix") for s in config["layers"][cut:]):
            return 0
        mx = config["layers"][j]["mixer"]
        return int(mx["kv_heads"]) * int(mx["vdim"])

    @property
    def hop_width(self) -> int:
        return (self.config.hidden_size
                + self.carried(self.config, self.shard.start_layer))

    def _key_optional(self, key: str) -> bool:
        # only layers with v_mix have one
        top, _, leaf = key.partition(".mix.")
        return leaf == "vmix" and not self.config["layers"][int(top[1:])][
            "mixer"].get("v_mix")

    # -- forward -----------------------------------------------------------
    @torch.no_grad()
    def run(self, x: torch.Tensor, batch: RaggedBatch, state: PagedState,
            rows: Optional[torch.Tensor] = None,
            layer_outputs: Optional[list] = None) -> torch.Tensor:
        W, cfg = self.config.hidden_size, self.config
        dtype = next(self.parameters()).dtype
        mult = float(cfg["residual_mult"])
        first = None
        if not self.shard.is_first and self.hop_width > W:
            first = x[:, W:].to(dtype)
        x = self.residual(x)
        items = self.layer_items()
        h = ragged.add_norm(x, None, None, items[0][1].norm1.weight, self.eps,
                            0.0, dtype)
        for k, (i, layer) in enumerate(items):
            y, v = layer(h, batch, state.layers[k],
                         first if layer.mixes else None)
            if i == self.first_mix(cfg):
                first = v
            after = None
            if k + 1 < len(items):
                after = items[k + 1][1].norm1.weight
            elif self.shard.is_last:
                after = self.final.norm.weight
            h = ragged.add_norm(x, y, None, after, self.eps, 0.0, dtype, mult)
            if layer_outputs is not None:
                layer_outputs.append(x.clone())
        if not self.shard.is_last:
            if self.carried(cfg, self.shard.end_layer):
                x = torch.cat([x, first.float()], 1)
            return x
        if rows is not None:
            h = h.index_select(0, rows)
        return ragged.cap_logits(self.head(h), float(cfg["logit_scale"]),
                                 float(cfg["logit_softcap"]))
