"""Causal convolutions over time and the selective scan on ragged batches.

The same policy as the other ragged ops: GPU tensors run the hand-written
kernels, CPU tensors plain torch, request by request, on the same storage.
What a request carries from step to step lies in its slot: the last inputs of a
convolution [history, channels] and the state of a scan [states, channels], both
with the channel running fastest.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch
import torch.nn.functional as F

from .paged import RaggedBatch
from .ragged import _ext, _pad, add_norm

MAX_TAPS = 8


def _conv_request(h, w, history, slot: int, fresh: bool):
    """Convolution of one request's rows h [n, C] (fp32); its history moves on."""
    n, taps = h.shape[0], w.shape[0]
    x = h
    if taps > 1:
        old = torch.zeros_like(history[slot]) if fresh else history[slot].clone()
        x = torch.cat([old, h])
        history[slot] = x[n:]
    return sum(w[j].float() * x[j: j + n].float() for j in range(taps))


def causal_conv(h, w, bias, history, batch: RaggedBatch, add: bool = False,
                silu: bool = False, pad_to: int = 1):
    """Rows h [N, C] (may be columns of wider rows) convolved over time per
    channel with w [taps, C], the last tap on the current token; ``history``
    [slots, taps - 1, C] holds what came before a portion.  Then the bias (if
    given), silu or the rows themselves added.  Returns [N, C], the rows padded
    with zeros to a multiple of ``pad_to`` columns."""
    N, C = h.shape
    if h.is_cuda:
        ext = _ext("causal_conv")
        out = torch.empty(N, _pad(C, pad_to), dtype=h.dtype, device=h.device)
        if batch.n_short:
            ext.conv_short(h, w, bias, history, out, batch.cu, batch.pos0,
                           batch.slots, batch.n_short, batch.short_tokens, add,
                           silu)
        if batch.n_long:
            ext.conv_long(h, w, bias, history, out, batch.cu, batch.pos0,
                          batch.slots, batch.tok_entry, batch.chunks,
                          batch.n_short, batch.n_long, batch.short_tokens, 0,
                          add, silu)
        return out
    out = h.new_zeros(N, _pad(C, pad_to))
    for t0, n, p0, held in batch.host:
        rows = h[t0: t0 + n]
        y = _conv_request(rows, w, history, held.slot, p0 == 0)
        if bias is not None:
            y = y + bias.float()
        if silu:
            y = F.silu(y)
        if add:
            y = y + rows.float()
        out[t0: t0 + n, :C] = y.to(h.dtype)
    return out


def norm_conv(x, y, w_post, w_next, eps: float, conv_w, history,
              batch: RaggedBatch, dtype: torch.dtype, pad_to: int = 1):
    """A sublayer boundary with a convolution behind the norm: x += y (normed
    first and weighted if w_post is given; y may be None), h = rms(x) * w_next,
    and the result is h + conv(h)."""
    if x.is_cuda:
        like = next(t for t in (w_post, w_next, y) if t is not None)
        ext = _ext("norm_conv")
        n, N, W = batch.short_tokens, batch.n_tokens, x.shape[1]
        if n and ext.norm_conv_fits(W, y):
            out = torch.empty(N, _pad(W, pad_to), dtype=like.dtype,
                              device=x.device)
            ext.norm_conv_short(x, y, w_post, w_next, eps, conv_w, history, out,
                                batch.cu, batch.pos0, batch.slots,
                                batch.n_short, n)
            if n < N:
                h = add_norm(x[n:], None if y is None else y[n:], w_post,
                             w_next, eps, 0.0, dtype)
                ext.conv_long(h, conv_w, None, history, out, batch.cu,
                              batch.pos0, batch.slots, batch.tok_entry,
                              batch.chunks, batch.n_short, batch.n_long, n, n,
                              True, False)
            return out
    h = add_norm(x, y, w_post, w_next, eps, 0.0, dtype)
    return causal_conv(h, conv_w, None, history, batch, add=True, pad_to=pad_to)


@dataclass(frozen=True)
class ScanShape:
    """Sizes of a selective scan.  A wave's lanes take neighbouring channels
    and, where there are many states, ``parts`` of them; states are padded with
    zeros to whole parts.  ``columns``: where step input, B and C begin in the
    rows of the projection that makes them."""
    channels: int
    states: int
    rank: int

    MAX = 512

    @property
    def part(self) -> int:
        return next((p for p in (8, 16) if self.states <= p), 32)

    @property
    def parts(self) -> int:
        p = 1
        while p * self.part < self.states:
            p *= 2
        return p

    @property
    def statesp(self) -> int:
        return self.part * self.parts

    @property
    def columns(self):
        r = _pad(self.rank, 8)
        return 0, r, r + self.statesp

    @property
    def width(self) -> int:
        return self.columns[2] + self.statesp


def selective_scan(x, z, dt, dt_bias, bc, A, D, state, sh: ScanShape,
                   batch: RaggedBatch):
    """Per channel c and state n: S <- exp(d A) S + d x B, y = sum_n S C + D x
    with d = softplus(dt + dt_bias); returns y * silu(z).

    x, z, dt [N, channels]; bc [N, width] holds B and C; A [states padded,
    channels], D and dt_bias [channels] are fp32; state [slots, 1, states
    padded, channels] moves on."""
    if x.is_cuda:
        ext = _ext("selective_scan")
        out = torch.empty(x.shape[0], sh.channels, dtype=x.dtype, device=x.device)
        sizes = (sh.part, sh.parts, sh.columns[1], sh.columns[2])
        if batch.n_short:
            ext.scan_short(x, z, dt, dt_bias, bc, A, D, state, out, batch.cu,
                           batch.pos0, batch.slots, batch.n_short,
                           batch.short_tokens, *sizes)
        if batch.n_long:
            ext.scan_long(x, z, dt, dt_bias, bc, A, D, state, out, batch.pos0,
                          batch.slots, batch.spans, batch.span_cu,
                          batch.n_short, batch.n_long, *sizes)
        return out
    out = x.new_empty(x.shape[0], sh.channels)
    b0, c0 = sh.columns[1:]
    for t0, n, p0, held in batch.host:
        at = slice(t0, t0 + n)
        xf, d = x[at].float(), F.softplus(dt[at].float() + dt_bias, threshold=80)
        B, C = (bc[at, c: c + sh.statesp].float() for c in (b0, c0))
        S = state[held.slot, 0]
        S = torch.zeros_like(S) if p0 == 0 else S.clone()
        y = torch.empty(n, sh.channels)
        for t in range(n):
            S = torch.exp(d[t] * A) * S + B[t][:, None] * (d[t] * xf[t])
            y[t] = (S * C[t][:, None]).sum(0)
        state[held.slot, 0] = S
        out[at] = ((y + D * xf) * F.silu(z[at].float())).to(x.dtype)
    return out
