"""Routed experts on ragged batches.

The router's choice stays on the device: tokens are sorted by expert into tiles
of one expert each, two grouped matrix products run the tiles, and every token
gathers what its experts gave.  Nothing waits for the host, so a captured graph
may hold all of it.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch
import torch.nn.functional as F

from .ragged import ClampedGLU, _ext, _pad

TILE_SHORT = 16    # tokens of one expert per tile where experts get few
TILE_LONG = 128
MAX_EXPERTS = 1024


@dataclass(frozen=True)
class ExpertShape:
    """``experts`` feed-forwards of ``ff`` units on rows of ``width``, and
    ``identity`` more that hand a row on as it is; a token uses ``top`` of
    them.  Contractions are padded with zeros to whole steps."""
    width: int
    ff: int
    experts: int
    identity: int
    top: int

    STEP = 64

    def __post_init__(self):
        if not 1 <= self.top <= self.total:
            raise ValueError(f"a token cannot use {self.top} of {self.total} "
                             f"experts")
        if self.total > MAX_EXPERTS:
            raise ValueError(f"{self.total} experts are above {MAX_EXPERTS}")

    @property
    def total(self) -> int:
        return self.experts + self.identity

    @property
    def widthp(self) -> int:
        return _pad(self.width, self.STEP)

    @property
    def ffp(self) -> int:
        return _pad(self.ff, self.STEP)

    def tile(self, tokens: int) -> int:
        few = tokens * self.top <= 48 * self.total
        return TILE_SHORT if few else TILE_LONG


def pack(w, width: int):
    """Weights [rows, columns], the columns padded to ``width``, as matrix-core
    operands of 16 rows by 32 columns, lane = (column / 8 % 4, row % 16)."""
    rows, cols = w.shape
    w = F.pad(w, (0, width - cols, 0, -rows % 16))
    w = w.view(-1, 16, width // 32, 4, 8).permute(0, 2, 3, 1, 4)
    return w.reshape(-1, width // 32, 64, 8).contiguous()


def unpack(w, rows: int, cols: int):
    w = w.view(-1, w.shape[1], 4, 16, 8).permute(0, 3, 1, 2, 4)
    return w.reshape(w.shape[0] * 16, -1)[:rows, :cols]


@dataclass(frozen=True)
class Routing:
    """How a router's logits become a choice and weights: ``score`` softmax or
    sigmoid; ``normalize``: the chosen scores are divided by their sum;
    ``on_input``: the weight multiplies what the expert reads, not what it
    gives."""
    score: str = "softmax"
    normalize: bool = True
    on_input: bool = False

    def __post_init__(self):
        if self.score not in ("softmax", "sigmoid"):
            raise ValueError(f"unknown router score {self.score!r}")


def route(h, router, correction, sh: ExpertShape, routing: Routing = Routing()):
    """Chosen experts [N, top] and their weights (fp32).  The choice is by
    score + correction (if there is one), the weights are the scores alone."""
    z = h[:, : sh.width].float() @ unpack(router, sh.total, sh.width).float().T
    s = torch.softmax(z, -1) if routing.score == "softmax" else torch.sigmoid(z)
    # logits order uncorrected scores, also where those round to the same
    by = z if correction is None else s + correction.float()
    idx = torch.topk(by, sh.top, dim=-1).indices
    w = s.gather(-1, idx)
    if routing.normalize:
        w = w / (w.sum(-1, keepdim=True) + 1e-20)
    return idx, w


def expert_rows(h, router, correction, up, down, sh: ExpertShape,
                routing: Routing = Routing(), glu: Optional[ClampedGLU] = None):
    """What the chosen experts make of rows h [N, width padded]: (rows, where
    [N, top] the rows of a token are (-1: an identity expert), weights [N, top]
    that they still have to be multiplied by, or None).

    An expert is W_down relu(W_up h)^2, or W_down glu(W_gate h, W_up h).  up
    [experts, ff padded, width padded], with the gate's rows before the up
    projection's if there is one; down [experts, width, ff padded]; router
    packed."""
    N = h.shape[0]
    if h.is_cuda:
        ext = _ext("experts")
        tile = sh.tile(N)
        idx, weight, rank, hist = ext.expert_route(
            h, router, correction, sh.total, sh.experts, sh.top,
            routing.score == "sigmoid", routing.normalize)
        scale = weight if routing.on_input else None
        where, tokens, tiles, scale = ext.expert_plan(idx, rank, hist, scale,
                                                      sh.experts, tile)
        form = (0.0, 0.0) if glu is None else (glu.limit, glu.alpha)
        u = ext.expert_gemm(h, tokens, tiles, up, scale, tile, N * sh.top,
                            1 if glu is None else 2, *form)
        d = ext.expert_gemm(u, None, tiles, down, None, tile, N * sh.top, 0,
                            0.0, 0.0)
        return d, where, None if routing.on_input else weight
    idx, weight = route(h, router, correction, sh, routing)
    d = h.new_zeros(N * sh.top, sh.width)
    where = torch.arange(N * sh.top).view(N, sh.top)
    where = where.masked_fill(idx >= sh.experts, -1).int()
    for e in range(sh.experts):
        tok, k = (idx == e).nonzero(as_tuple=True)
        if not tok.numel():
            continue
        u = h[tok].float() @ up[e].float().T
        if routing.on_input:
            u = u * weight[tok, k, None]
        if glu is None:
            u = u.clamp(min=0).square()
        else:
            u = glu.of(*u.chunk(2, -1))
        d[tok * sh.top + k] = (u.to(h.dtype).float()
                               @ down[e].float().T).to(h.dtype)
    return d, where, None if routing.on_input else weight


def add_experts(x, h, router, correction, up, down, sh: ExpertShape,
                copy: bool = False, routing: Routing = Routing(),
                glu: Optional[ClampedGLU] = None):
    """x [N, width] (fp32) += the weighted sum of the chosen experts of rows h
    (operands as above).  copy: returns x in h's type as well."""
    if routing.on_input and sh.identity:
        raise ValueError("identity experts have no input to weigh")
    d, where, weight = expert_rows(h, router, correction, up, down, sh, routing,
                                   glu)
    if weight is None:
        weight = torch.ones(where.shape, device=x.device)
    if x.is_cuda:
        return _ext("experts").expert_combine(x, h, d, where, weight, copy)
    rows = torch.where((where < 0)[..., None], h[:, None, : sh.width],
                       d[where.long()])
    x += (weight[..., None] * rows.float()).sum(1)
    return x.to(h.dtype) if copy else None


FEW = 64  # rows that one skinny product takes


def token_gate(x, gate, e):
    """gelu_tanh(gate x) * e for a few rows of the fp32 residual x, in one
    kernel; gate packed."""
    return _ext("token_gate").token_gate(x, gate, e)
