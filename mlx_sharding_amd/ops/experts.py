"""Routed experts on ragged batches.

The router's choice stays on the device: tokens are sorted by expert into tiles
of one expert each, two grouped matrix products run the tiles, and every token
gathers what its experts gave.  Nothing waits for the host, so a captured graph
may hold all of it.
"""

from __future__ import annotations

from dataclasses import dataclass

import torch
import torch.nn.functional as F

from .ragged import _ext, _pad

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


def route(h, router, correction, sh: ExpertShape):
    """Softmax router: chosen experts [N, top] and their weights (fp32).  The
    choice is by score + correction, the weights are the scores alone, divided
    by their sum."""
    z = h[:, : sh.width].float() @ unpack(router, sh.total, sh.width).float().T
    s = torch.softmax(z, -1)
    idx = torch.topk(s + correction.float(), sh.top, dim=-1).indices
    w = s.gather(-1, idx)
    return idx, w / (w.sum(-1, keepdim=True) + 1e-20)


def add_experts(x, h, router, correction, up, down, sh: ExpertShape,
                copy: bool = False):
    """x [N, width] (fp32) += the weighted sum of the chosen experts of rows h
    [N, width padded], each W_down relu(W_up h)^2.  up [experts, ff padded,
    width padded], down [experts, width, ff padded], router packed.  copy: returns x in h's type as well."""
    if x.is_cuda:
        ext = _ext("experts")
        N = x.shape[0]
        tile = sh.tile(N)
        idx, weight, rank, hist = ext.expert_route(h, router, correction,
                                                   sh.experts, sh.top)
        where, tokens, tiles = ext.expert_plan(idx, rank, hist, sh.experts, tile)
        u = ext.expert_gemm(h, tokens, tiles, up, tile, N * sh.top, True)
        d = ext.expert_gemm(u, None, tiles, down, tile, N * sh.top, False)
        return ext.expert_combine(x, h, d, where, weight, copy)
    idx, weight = route(h, router, correction, sh)
    hf = h[:, : sh.width].float()
    y = torch.zeros_like(x)
    for e in range(sh.total):
        tok, k = (idx == e).nonzero(as_tuple=True)
        if not tok.numel():
            continue
        v = hf[tok]
        if e < sh.experts:
            u = (h[tok].float() @ up[e].float().T).clamp(min=0).square()
            v = u.to(h.dtype).float() @ down[e].float().T
        y.index_add_(0, tok, weight[tok, k, None] * v)
    x += y
    return x.to(h.dtype) if copy else None


FEW = 64  # rows that one skinny product takes


def token_gate(x, gate, e):
    """gelu_tanh(gate x) * e for a few rows of the fp32 residual x, in one
    kernel; gate packed."""
    return _ext("token_gate").token_gate(x, gate, e)
