"""Ops on ragged batches: HIP kernels on GPU, torch on CPU.

The same policy as the package's other ops: GPU tensors run the hand-written
kernels (extension ``_hip_ragged``) or fail loudly; CPU tensors run plain torch
with the same storage layout, request by request.

Layouts.  A latent row is [latent, zero padding to ``rankp`` | rotated key part,
zero padding to ``rotp``].  A query head is [unrotated, padding | rotated,
padding], ``dq`` wide.

A page of keys and values holds, for each key/value head, 64 keys and then 64
values in the order in which the matrix cores take them: tiles of 16 x 32
elements, a lane's 8 elements together, lane after lane.  A key tile is 16 keys
by 32 dimensions, lane = (dimension / 8 % 4, key % 16).  A value tile is 16
dimensions by 32 keys, lane = (key / 4 % 4, dimension % 16), and a lane's
elements are keys 0..3 and 16..19 past its first.
"""

from __future__ import annotations

import math
from dataclasses import dataclass
from typing import List, Optional, Tuple

import torch
import torch.nn.functional as F

from .paged import LayerStore, PAGE, RaggedBatch

_EXT = None
_EXT_ERR: Optional[str] = None
_TRIED = False


def hip_ragged():
    """The extension module, or None where it is not built."""
    global _EXT, _EXT_ERR, _TRIED
    if not _TRIED:
        _TRIED = True
        try:
            from mlx_sharding_amd import _hip_ragged
            _EXT = _hip_ragged
        except ImportError as e:
            _EXT_ERR = repr(e)
    return _EXT


def _ext(op: str):
    ext = hip_ragged()
    if ext is None:
        raise RuntimeError(
            f"mlx_sharding_amd: op '{op}' called on a GPU tensor but the HIP "
            f"extension mlx_sharding_amd._hip_ragged is not importable "
            f"({_EXT_ERR}). Build it with `python setup.py build_ext --inplace`.")
    return ext


def _pad(n: int, to: int) -> int:
    return (n + to - 1) // to * to


# ---------------------------------------------------------------------------
# Norms around a 32-bit residual
# ---------------------------------------------------------------------------

def _rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def add_norm(x, y, w_post, w_next, eps: float, offset: float,
             dtype: torch.dtype, mult: float = 1.0, *, where=None, y_bias=None,
             copy: bool = False, pad_to: int = 1):
    """x += mult * rms(y) * (w_post + offset), in place, if y is given (without
    w_post: x += mult * y); returns rms(x) * (w_next + offset) in ``dtype``, or
    None without w_next.  x is the fp32 residual [N, W].

    where [N, top]: row i of y is the sum of the rows y[where[i]].  y_bias [W] is
    added to y's rows before all else.  copy: without
    w_next, returns x itself in ``dtype``.  What is returned is padded with
    zeros to a multiple of ``pad_to`` columns."""
    wide = _pad(x.shape[1], pad_to)
    if x.is_cuda:
        out = w_next is not None or copy
        h = _ext("add_norm").add_norm(x, y, w_post, w_next,
                                      dtype == torch.float32, eps, offset,
                                      mult, where, wide if out else 0, y_bias)
        return h if out else None
    if y is not None:
        y = y.float() if where is None else y[where.long()].float().sum(1)
        y = y[:, : x.shape[1]]
        if y_bias is not None:
            y = y + y_bias.float()
        if w_post is not None:
            y = _rms(y, eps) * (w_post.float() + offset)
        x += mult * y
    if w_next is None:
        if not copy:
            return None
        h = x
    else:
        h = _rms(x, eps) * (w_next.float() + offset)
    return F.pad(h, (0, wide - h.shape[1])).to(dtype, copy=True)


# ---------------------------------------------------------------------------
# Rotation tables
# ---------------------------------------------------------------------------

@dataclass(frozen=True)
class Rotary:
    """Interleaved rotary positions on ``dims`` dimensions, optionally with
    YaRN frequencies (``factor`` set): pairs that turn less than ``slow`` times
    within ``original`` positions are slowed by ``factor``, pairs that turn more
    than ``fast`` times are kept, with a ramp between; cos and sin are scaled
    by 0.1 ln(factor) + 1."""
    dims: int
    base: float
    factor: Optional[float] = None
    original: float = 4096
    fast: float = 32.0
    slow: float = 1.0

    def frequencies(self) -> torch.Tensor:
        i = torch.arange(self.dims // 2, dtype=torch.float64)
        f = self.base ** (-2.0 * i / self.dims)
        if self.factor is None:
            return f

        def dim_of(turns):
            return (self.dims * math.log(self.original / (2 * math.pi * turns))
                    / (2 * math.log(self.base)))

        lo = max(math.floor(dim_of(self.fast)), 0)
        hi = min(math.ceil(dim_of(self.slow)), self.dims - 1)
        ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
        return f / self.factor * ramp + f * (1.0 - ramp)

    @property
    def magnitude(self) -> float:
        return 1.0 if self.factor is None else 0.1 * math.log(self.factor) + 1.0

    def tables(self, n: int, device):
        """cos, sin [n, dims / 2], fp32."""
        a = torch.arange(n, dtype=torch.float64)[:, None] * self.frequencies()
        return ((torch.cos(a) * self.magnitude).float().to(device).contiguous(),
                (torch.sin(a) * self.magnitude).float().to(device).contiguous())


# ---------------------------------------------------------------------------
# Latent attention
# ---------------------------------------------------------------------------

@dataclass(frozen=True)
class LatentShape:
    """Sizes of a latent-attention layer, and how they are padded: what the
    kernels see are multiples of their tiles, filled with zeros."""
    heads: int
    dim: int
    rot: int
    vdim: int
    rank: int
    f32: bool = False

    @property
    def dimp(self):
        return _pad(self.dim, 32)

    @property
    def rotp(self):
        return _pad(self.rot, 32)

    @property
    def dq(self):
        return self.dimp + self.rotp

    @property
    def rankp(self):
        p = 64
        while p < self.rank:
            p *= 2
        return p

    @property
    def width(self):
        """Elements of a cached row."""
        return self.rankp + self.rotp

    @property
    def vdp(self):
        for p in ((64, 256) if self.f32 else (32, 64, 128, 256)):
            if self.vdim <= p:
                return p
        return _pad(self.vdim, 16)

    @property
    def expandable(self) -> bool:
        """Whether the expanded kernel has this head shape; otherwise every
        portion takes the absorbed one."""
        return self.dq <= 256 and self.vdim <= 256


def latent_append(dkv, norm_w, eps: float, store: LayerStore, q, sh: LatentShape,
                  cos, sin, batch: RaggedBatch):
    """Rotate the queries [N, heads * dq] in place and, unless dkv is None (the
    layer reads another layer's rows), write this batch's latent rows."""
    if q.is_cuda:
        _ext("latent_append").latent_append(
            dkv, norm_w, eps, store.rows, q, sh.heads, sh.dq, sh.dimp, sh.rank,
            sh.rankp, sh.rot, sh.rotp, cos, sin, batch.tok_pos,
            batch.tok_entry, batch.pages)
        return
    pos = batch.tok_pos.long()
    c, s = cos[pos], sin[pos]

    def turn(x, c, s):
        u, v = x[..., 0::2].float(), x[..., 1::2].float()
        return torch.stack([u * c - v * s, v * c + u * s], -1).flatten(-2).to(x.dtype)

    qh = q.view(q.shape[0], -1)[:, : sh.heads * sh.dq].unflatten(1, (sh.heads, sh.dq))
    part = qh[..., sh.dimp: sh.dimp + sh.rot]
    part.copy_(turn(part, c[:, None], s[:, None]))
    if dkv is None:
        return
    pages = batch.pages[batch.tok_entry.long(), pos // PAGE].long()
    row = torch.zeros(q.shape[0], sh.width, dtype=store.rows.dtype)
    row[:, : sh.rank] = (_rms(dkv[:, : sh.rank].float(), eps)
                         * norm_w.float()).to(row.dtype)
    row[:, sh.rankp: sh.rankp + sh.rot] = turn(
        dkv[:, sh.rank: sh.rank + sh.rot], c, s).to(row.dtype)
    store.rows[pages * PAGE + pos % PAGE] = row


def latent_attention_absorbed(q, q_abs, store: LayerStore, sh: LatentShape,
                              scale: float, batch: RaggedBatch, n_req: int,
                              max_len: int):
    """Attention of the first n_req requests over the cached rows themselves.
    q_abs [heads, tokens, rankp]; returns the same shape."""
    if q.is_cuda:
        return _ext("latent_attn_short").latent_attn_short(
            q_abs, q, store.rows, batch.cu, batch.pos0, batch.pages, n_req,
            max_len, batch.max_keys, sh.dq, sh.dimp, sh.rotp, scale)
    out = torch.zeros_like(q_abs)
    for t0, n, p0, held in batch.host[:n_req]:
        rows = _gather_rows(store, held, p0 + n)
        qr = q[t0: t0 + n, : sh.heads * sh.dq].unflatten(1, (sh.heads, sh.dq))
        qf = torch.cat([q_abs[:, t0: t0 + n].float(),
                        qr[..., sh.dimp:].transpose(0, 1).float()], -1)
        s = (qf @ rows.float().T) * scale
        dead = torch.arange(p0 + n)[None, :] > torch.arange(p0, p0 + n)[:, None]
        p = torch.softmax(s.masked_fill(dead, float("-inf")), -1)
        out[:, t0: t0 + n] = (p @ rows[:, : sh.rankp].float()).to(out.dtype)
    return out


def _gather_rows(store: LayerStore, held, n: int) -> torch.Tensor:
    pages = torch.tensor(held.pages, dtype=torch.long)
    idx = (pages[:, None] * PAGE + torch.arange(PAGE)[None, :]).reshape(-1)[:n]
    return store.rows[idx]


def latent_attention_expanded(q, store: LayerStore, w_uk, w_uv, sh: LatentShape,
                              scale: float, batch: RaggedBatch):
    """Attention of the long portions: keys and values of their whole prefix
    are expanded from the gathered rows.  w_uk [heads * dimp, rankp], w_uv
    [heads * vdp, rankp]; returns [long tokens, heads * vdp]."""
    if q.is_cuda:
        ext = _ext("latent_attn_long")
        lat = ext.latent_gather(store.rows, batch.blocks, batch.key_rows)
        c = lat[:, : sh.rankp]
        kx = F.linear(c, w_uk)
        vt = F.linear(w_uv, c)  # already transposed: [heads * vdp, keys]
        return ext.latent_attn_long(
            q, kx, lat, vt, batch.tiles, batch.cu, batch.pos0, batch.cuk,
            batch.n_short, batch.short_tokens, sh.heads, sh.dimp, sh.rotp,
            scale)
    base = batch.short_tokens
    out = q.new_zeros(batch.n_tokens - base, sh.heads * sh.vdp)
    for t0, n, p0, held in batch.host[batch.n_short:]:
        rows = _gather_rows(store, held, p0 + n).float()
        c = rows[:, : sh.rankp]
        k = (c @ w_uk.float().T).unflatten(1, (sh.heads, sh.dimp))
        v = (c @ w_uv.float().T).unflatten(1, (sh.heads, sh.vdp))
        qh = q[t0: t0 + n, : sh.heads * sh.dq].unflatten(1, (sh.heads, sh.dq)).float()
        s = torch.matmul(qh[..., : sh.dimp].transpose(0, 1), k.permute(1, 2, 0))
        s = s + torch.matmul(qh[..., sh.dimp:].transpose(0, 1), rows[:, sh.rankp:].T)
        dead = torch.arange(p0 + n)[None, :] > torch.arange(p0, p0 + n)[:, None]
        p = torch.softmax((s * scale).masked_fill(dead, float("-inf")), -1)
        o = torch.matmul(p, v.transpose(0, 1)).transpose(0, 1)
        out[t0 - base: t0 - base + n] = o.flatten(1).to(out.dtype)
    return out


# ---------------------------------------------------------------------------
# Grouped attention
# ---------------------------------------------------------------------------

@dataclass(frozen=True)
class GroupedShape:
    """Sizes of a grouped-attention layer; heads are padded to whole tiles."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int

    MAX = 512    # largest head size
    LONG = 256   # largest head size of the prompt kernel

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} heads do not share "
                             f"{self.kv_heads} key/value heads evenly")

    @property
    def dimp(self):
        return _pad(self.dim, 32)

    @property
    def vdp(self):
        return _pad(self.vdim, 16)

    @property
    def width(self):
        """Cached elements per token."""
        return self.kv_heads * (self.dimp + self.vdp)

    @property
    def prompts(self) -> bool:
        """Whether the prompt kernel has this head shape; otherwise every
        portion takes the decode kernel."""
        return max(self.dimp, self.vdp) <= self.LONG

    def keys(self, rows):
        """A view of a page pool: [page, key / 16, key % 16, head, ...] with
        the last dimensions a head's key in order."""
        p = rows.view(-1, self.kv_heads, PAGE * (self.dimp + self.vdp))
        k = p[..., : PAGE * self.dimp].unflatten(
            2, (PAGE // 16, self.dimp // 32, 4, 16, 8))
        return k.permute(0, 2, 5, 1, 3, 4, 6)

    def values(self, rows):
        """[page, key / 32, key / 16 % 2, key / 4 % 4, key % 4, head, ...]."""
        p = rows.view(-1, self.kv_heads, PAGE * (self.dimp + self.vdp))
        v = p[..., PAGE * self.dimp:].unflatten(
            2, (self.vdp // 16, PAGE // 32, 4, 16, 2, 4))
        return v.permute(0, 3, 6, 4, 7, 1, 2, 5)


@dataclass
class Turns:
    """Rotations of grouped attention, as (cos, sin) tables [positions, pairs]
    over neighbouring pairs.  ``qk``: on the first dimensions of queries and
    keys.  ``v``: over whole values; each head's output is turned back by its
    own position, so that only the distance to a value's token counts."""
    qk: Optional[Tuple[torch.Tensor, torch.Tensor]] = None
    v: Optional[Tuple[torch.Tensor, torch.Tensor]] = None


def _turn(x, table, pos, sign: float = 1.0):
    """x [N, heads, size] with its first pairs rotated, fp32."""
    c, s = table[0][pos][:, None], sign * table[1][pos][:, None]
    n = 2 * c.shape[-1]
    u, v = x[..., 0:n:2].float(), x[..., 1:n:2].float()
    turned = torch.stack([u * c - v * s, v * c + u * s], -1).flatten(-2)
    return torch.cat([turned, x[..., n:].float()], -1)


def grouped_append(y, wq, wk, eps: float, vmix, first, store: LayerStore,
                   sh: GroupedShape, batch: RaggedBatch,
                   turns: Optional[Turns] = None, head_norm: bool = False,
                   own: bool = True):
    """From projection rows y [N, q | k | v | ...]: the queries [N, heads,
    dimp], RMS-normed over the row if wq is given; keys (normed likewise) and
    values go to their pages.  first: values [N, kv_heads * vdim] that are
    blended in by vmix (one element).  turns: rotations by position.
    head_norm: every query and key is divided by its own root mean square
    (before it is rotated), and wq, wk are weights [dim] that all heads share.
    own: otherwise y is [N, q | ...] and nothing is written."""
    H, G, D, V = sh.heads, sh.kv_heads, sh.dim, sh.vdim
    by_head = head_norm or turns is not None or not own
    if by_head and first is not None:
        raise ValueError("rotations and norms per head do not go together with "
                         "blended values")
    if by_head and not head_norm and not (wq is None and wk is None):
        raise ValueError("rotations do not go together with norms over whole "
                         "rows")
    turns = turns or Turns()
    if y.is_cuda:
        ext = _ext("grouped_append")
        direct = batch.short_tokens if sh.prompts else batch.n_tokens
        tables = (*(turns.qk or (None, None)), *(turns.v or (None, None)))
        if by_head:
            q, kinv = ext.grouped_turn(
                y, wq, wk, eps, head_norm, *tables, store.rows, H, G, D, V,
                sh.dimp, sh.vdp, batch.tok_pos, batch.tok_entry, batch.pages,
                direct, own)
        else:
            q, kinv = ext.grouped_append(
                y, wq, wk, eps, vmix, first, store.rows, H, G, D, V, sh.dimp,
                sh.vdp, batch.tok_pos, batch.tok_entry, batch.pages, direct)
        if own and direct < batch.n_tokens:
            ext.grouped_fill(y, wk, kinv, vmix, first, store.rows, H, G, D, V,
                             sh.dimp, sh.vdp, batch.fills, head_norm, *tables,
                             batch.tok_pos)
        return q
    N = y.shape[0]
    pos = batch.tok_pos.long()

    def ready(x, w, heads):
        if not head_norm and w is not None:
            x = _rms(x, eps) * w.float()
        x = x.view(N, heads, D)
        if head_norm:
            x = _rms(x, eps)
            x = x if w is None else x * w.float()
        if turns.qk is not None:
            x = _turn(x, turns.qk, pos)
        return F.pad(x, (0, sh.dimp - D)).to(y.dtype)

    q = ready(y[:, : H * D].float(), wq, H)
    if not own:
        return q
    k, v = (t.float() for t in y[:, H * D: (H + G) * D + G * V].split(
        [G * D, G * V], 1))
    k = ready(k, wk, G)
    if first is not None:
        lam = vmix.float()
        v = (1.0 - lam) * v + lam * first.float()
    v = v.view(N, G, V)
    if turns.v is not None:
        v = _turn(v, turns.v, pos)
    v = F.pad(v, (0, sh.vdp - V)).to(y.dtype)
    page, r = batch.pages[batch.tok_entry.long(), pos // PAGE].long(), pos % PAGE
    sh.keys(store.rows)[page, r // 16, r % 16] = k.view(N, G, -1, 4, 8)
    sh.values(store.rows)[page, r // 32, r // 16 % 2, r // 4 % 4, r % 4] = \
        v.view(N, G, -1, 16)
    return q


def grouped_attention(q, sink, store: LayerStore, sh: GroupedShape,
                      scale: float, batch: RaggedBatch, out,
                      window: Optional[int] = None,
                      turns: Optional[Turns] = None, gate=None):
    """Attention of queries [N, heads, dimp] over their requests' pages, into
    out [N, heads * vdim].  sink [heads] (or None): a score per head that only
    the softmax's denominator sees.  window: how many tokens a token sees, up
    to itself (None: all).  turns: where values are rotated, the output is
    turned back.  gate [N, heads] (may be columns of wider rows): every head's
    output is multiplied by the sigmoid of its number."""
    back = turns.v if turns is not None else None
    if q.is_cuda:
        ext = _ext("grouped_attention")
        n_req, n, max_len = batch.n_short, batch.short_tokens, batch.max_short
        if not sh.prompts:
            n_req, n, max_len = batch.n_requests, batch.n_tokens, batch.max_len
        more = (window or 0, *(back or (None, None)), batch.tok_pos, gate)
        if n_req:
            ext.grouped_attn_short(
                q, sink, store.rows, out, batch.cu, batch.pos0, batch.pages,
                n_req, n, max_len, batch.max_keys, sh.kv_heads, sh.vdim,
                sh.vdp, scale, *more)
        if n_req < batch.n_requests:
            ext.grouped_attn_long(
                q, sink, store.rows, out, batch.tiles, batch.cu, batch.pos0,
                batch.pages, sh.kv_heads, sh.vdim, sh.vdp, scale, *more)
        return
    H, G = sh.heads, sh.kv_heads
    for t0, n, p0, held in batch.host:
        S = p0 + n
        pages = torch.tensor(held.pages, dtype=torch.long)[: (S + PAGE - 1) // PAGE]
        k = sh.keys(store.rows)[pages].reshape(-1, G, sh.dimp)[:S].float()
        v = sh.values(store.rows)[pages].reshape(-1, G, sh.vdp)[:S].float()
        qg = q[t0: t0 + n].float().view(n, G, H // G, sh.dimp)
        s = torch.matmul(qg.permute(1, 2, 0, 3), k.permute(1, 2, 0)[:, None])
        at = torch.arange(p0, S)
        gap = at[:, None] - torch.arange(S)[None, :]
        dead = gap < 0 if window is None else (gap < 0) | (gap >= window)
        s = (s * scale).masked_fill(dead, float("-inf"))
        if sink is not None:
            extra = sink.float().view(G, H // G, 1, 1).expand(-1, -1, n, -1)
            s = torch.cat([s, extra], -1)
        p = torch.softmax(s, -1)[..., :S]
        o = torch.matmul(p, v.transpose(0, 1)[:, None])[..., : sh.vdim]
        o = o.permute(2, 0, 1, 3).reshape(n, H, sh.vdim)
        if back is not None:
            o = _turn(o, back, at, -1.0)
        if gate is not None:
            o = o * torch.sigmoid(gate[t0: t0 + n].float())[..., None]
        out[t0: t0 + n] = o.reshape(n, -1).to(out.dtype)


# ---------------------------------------------------------------------------
# Row-wise functions
# ---------------------------------------------------------------------------

def gelu(x, out=None):
    """The exact (erf) gelu of rows [..., C]; out may be a column slice."""
    if out is None:
        out = torch.empty(x.shape, dtype=x.dtype, device=x.device)
    if x.is_cuda:
        _ext("gelu").gelu(x.view(-1, x.shape[-1]), out.view(-1, x.shape[-1]))
    else:
        out.copy_(F.gelu(x.float()))
    return out


@dataclass(frozen=True)
class ClampedGLU:
    """g sigmoid(alpha g) (u + 1) with g = min(gate, limit) and u = up within
    +-limit."""
    limit: float
    alpha: float = 1.702

    def __call__(self, gate, up, gate_bias=None, up_bias=None):
        """Rows [N, C], which may be columns of wider ones; biases [C] are
        added first."""
        if gate.is_cuda:
            return _ext("clamped_glu").clamped_glu(gate, up, self.limit,
                                                   self.alpha, gate_bias, up_bias)
        g, u = gate.float(), up.float()
        if gate_bias is not None:
            g = g + gate_bias.float()
        if up_bias is not None:
            u = u + up_bias.float()
        return self.of(g, u).to(gate.dtype)

    def of(self, gate, up):
        g, u = gate.clamp(max=self.limit), up.clamp(-self.limit, self.limit)
        return g * torch.sigmoid(self.alpha * g) * (u + 1.0)


def cap_logits(z, scale: float, limit: float):
    """limit * tanh(z * scale / limit), fp32."""
    if z.is_cuda:
        return _ext("cap_logits").cap_logits(z, scale, limit)
    return limit * torch.tanh(z.float() * scale / limit)


# ---------------------------------------------------------------------------
# Gated delta rule
# ---------------------------------------------------------------------------

@dataclass(frozen=True)
class DeltaShape:
    """Sizes of a gated-delta layer and the columns of its projection row
    [q | k | v | gate | decay | beta].

    ``ranks``: one decay per head and key channel, and decay and gate are made
    by a second projection of (decay, gate) ``ranks`` columns each.  The row is
    [q | k | v | decay inputs | gate inputs | beta] then, inputs from whole
    vectors on, and a second one [decay | gate] has what comes of them."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int
    ranks: Optional[Tuple[int, int]] = None

    @property
    def widths(self) -> List[int]:
        k, v = self.kv_heads * self.dim, self.heads * self.vdim
        if self.ranks is None:
            return [k, k, v, v, self.heads, self.heads]
        return [k, k, v, *self.ranks, self.heads]

    @property
    def columns(self) -> List[int]:
        out, at = [], 0
        for i, w in enumerate(self.widths):
            if self.ranks is not None and i >= 3:
                at = _pad(at, 8)
            out.append(at)
            at += w
        return out

    @property
    def inputs(self) -> Tuple[int, int]:
        """Columns of the inputs of the second projection, from and to."""
        at = self.columns
        return at[3], at[5]

    @property
    def places(self) -> List[int]:
        """Columns of q, k, v, gate, decay and beta, each in its row."""
        at = self.columns
        if self.ranks is not None:
            at = [*at[:3], self.heads * self.dim, 0, at[5]]
        return at

    @property
    def channels(self) -> int:
        """Channels behind a short convolution: q, k and v."""
        return sum(self.widths[:3])


def gated_delta(y, conv_w, A_log, dt_bias, norm_w, store: LayerStore,
                sh: DeltaShape, eps: float, batch: RaggedBatch, z=None,
                sigmoid_gate: bool = False):
    """Projection rows y [N, *] -> [N, heads * vdim]; state and convolution
    inputs of every request move on.  z: the second rows of a shape with
    ``ranks``.  The output gate is silu, or sigmoid if asked for."""
    if y.is_cuda:
        ext = _ext("gated_delta")
        out = torch.empty(y.shape[0], sh.heads * sh.vdim, dtype=y.dtype,
                          device=y.device)
        more = (sh.kv_heads, sh.heads, sh.dim, sh.vdim, sh.places, eps, z,
                sigmoid_gate)
        if batch.n_short:
            ext.delta_short(y, conv_w, A_log, dt_bias, norm_w, store.state,
                            store.conv, out, batch.cu, batch.pos0, batch.slots,
                            batch.n_short, batch.max_short, *more)
        if batch.n_long:
            ext.delta_long(y, conv_w, A_log, dt_bias, norm_w, store.state,
                           store.conv, out, batch.cu, batch.pos0, batch.slots,
                           batch.tok_entry, batch.chunks, batch.chunk_cu,
                           batch.n_short, batch.n_long, batch.short_tokens,
                           *more)
        return out
    out = y.new_empty(y.shape[0], sh.heads * sh.vdim)
    for t0, n, p0, held in batch.host:
        out[t0: t0 + n] = _gated_delta_request(
            y[t0: t0 + n], None if z is None else z[t0: t0 + n], conv_w, A_log,
            dt_bias, norm_w, store, held.slot, p0 == 0, sh, eps, sigmoid_gate)
    return out


def _gated_delta_request(y, z, conv_w, A_log, dt_bias, norm_w, store, slot: int,
                         fresh: bool, sh: DeltaShape, eps: float,
                         sigmoid_gate: bool):
    n, hist = y.shape[0], sh.taps - 1
    H, KH, D, V = sh.heads, sh.kv_heads, sh.dim, sh.vdim
    old = torch.zeros_like(store.conv[slot]) if fresh else store.conv[slot]
    x = torch.cat([old, y[:, : sh.channels].T], 1)       # [C, hist + n]
    store.conv[slot] = x[:, n:]
    c = F.silu((x.float().unfold(1, sh.taps, 1) * conv_w.float()[:, None, :]).sum(-1)).T
    q, k, v = c.split(sh.widths[:3], 1)
    gc, ac, bc = sh.places[3:]
    rows, steps = (y, 1) if z is None else (z, D)     # decays per head
    gate, a = (rows[:, i: i + w].float()
               for i, w in ((gc, H * V), (ac, H * steps)))
    beta = torch.sigmoid(y[:, bc: bc + H].float())

    def unit(t):
        t = t.reshape(n, KH, D)
        t = t / torch.sqrt(t.pow(2).sum(-1, keepdim=True) + 1e-6)
        return t.repeat_interleave(H // KH, 1)

    q, k, v = unit(q) * D ** -0.5, unit(k), v.reshape(n, H, V)
    step = F.softplus(a + dt_bias.float(), threshold=80).view(n, H, steps)
    g = torch.exp(-torch.exp(A_log.float())[:, None] * step)[..., None]
    S = torch.zeros_like(store.state[slot]) if fresh else store.state[slot].clone()
    o = torch.empty(n, H, V)
    for t in range(n):
        S *= g[t]
        u = beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
        S += k[t][:, :, None] * u[:, None, :]
        o[t] = torch.einsum("hdv,hd->hv", S, q[t])
    store.state[slot] = S
    act = torch.sigmoid if sigmoid_gate else F.silu
    o = _rms(o, eps) * norm_w.float() * act(gate).reshape(n, H, V)
    return o.reshape(n, H * V).to(y.dtype)
