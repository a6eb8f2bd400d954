"""Token mixers and layer pieces for ragged batches.

A mixer works on rows [tokens, width] of a ragged batch (ops.paged) and keeps
what it needs between steps in its layer's store.  Every constant is a
parameter, so designs combine them freely.  Parameters keep the checkpoint's
shapes; ``prepare`` lays them out for the kernels (sibling projections in one
GEMM, head sizes padded to the kernels' tiles) once they are on their device.
"""

from __future__ import annotations

from typing import Optional, Tuple

import torch
import torch.nn as nn
import torch.nn.functional as F

from .. import ops
from ..ops import experts, ragged, recurrent
from ..ops.experts import ExpertShape, Routing
from ..ops.paged import (HistorySpec, LayerSpec, LayerStore, RaggedBatch,
                         RowSpec, StateSpec)
from ..ops.ragged import (ClampedGLU, DeltaShape, GroupedShape, LatentShape,
                          Rotary, Turns)
from ..ops.recurrent import ScanShape
from .base import Linear, RMSNorm


def _param(*shape, dtype) -> nn.Parameter:
    return nn.Parameter(torch.empty(shape, dtype=dtype), requires_grad=False)


def _share(weight: torch.Tensor, *linears: Linear):
    """Make the linears' weights views of the stacked one."""
    off = 0
    for lin in linears:
        lin.weight.data = weight[off: off + lin.out_features]
        off += lin.out_features


class _Weight(nn.Module):
    def __init__(self, *shape, dtype):
        super().__init__()
        self.weight = _param(*shape, dtype=dtype)


class _Biased(_Weight):
    """A weight with a vector ``b``."""

    def __init__(self, *shape, dtype):
        super().__init__(*shape, dtype=dtype)
        self.b = _param(shape[0], dtype=dtype)


class CausalConv(nn.Module):
    """A causal convolution over time per channel, ``weight`` [channels, taps],
    the last tap on the current token, and a bias ``b`` if asked for."""

    def __init__(self, channels: int, taps: int, bias: bool,
                 dtype: torch.dtype):
        super().__init__()
        if not 1 <= taps <= recurrent.MAX_TAPS:
            raise ValueError(f"convolutions have 1 to {recurrent.MAX_TAPS} "
                             f"taps, not {taps}")
        self.weight = _param(channels, taps, dtype=dtype)
        self.b = _param(channels, dtype=dtype) if bias else None
        self._by_tap = None

    def prepare(self):
        self._by_tap = self.weight.data.T.contiguous()

    @property
    def by_tap(self) -> torch.Tensor:
        """[taps, channels], as the kernels read it."""
        if self._by_tap is None:
            self.prepare()
        return self._by_tap

    def history(self) -> HistorySpec:
        channels, taps = self.weight.shape
        return HistorySpec(channels, taps - 1)


class ScalarNorm(nn.Module):
    """An RMS norm whose weight is one number."""

    def __init__(self, dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        self.weight = _param(dtype=dtype)


class ConvLinear(Linear):
    """A projection followed by a causal convolution over time per channel,
    ``conv.weight`` [channels, taps], the last tap on the current token."""

    def __init__(self, in_features: int, out_features: int, taps: int,
                 dtype: torch.dtype):
        super().__init__(in_features, out_features, dtype=dtype)
        self.conv = _Weight(out_features, taps, dtype=dtype)


class NormedLinear(Linear):
    """A projection whose leading outputs are RMS-normed (``norm.weight``)."""

    def __init__(self, in_features: int, out_features: int, normed: int,
                 eps: float, dtype: torch.dtype):
        super().__init__(in_features, out_features, dtype=dtype)
        self.norm = RMSNorm(normed, eps, dtype=dtype)


class LatentAttention(nn.Module):
    """Causal softmax attention over a cached low-rank latent.

    Cached per token: the normed latent (``rank``) and one rotated key part
    shared by all heads (``rotary.dims``).  Keys are [W_uk c | rotated part],
    values W_uv c.  Without ``own_rows`` the layer has no latent projection and
    attends to the rows of another layer's store.
    """

    def __init__(self, width: int, heads: int, dim: int, vdim: int, rank: int,
                 rotary: Rotary, scale: float, eps: float,
                 own_rows: bool = True, dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        self.rotary, self.scale, self.eps = rotary, float(scale), eps
        self.sizes = dict(heads=heads, dim=dim, rot=rotary.dims, vdim=vdim,
                          rank=rank)
        if rank > 1024:
            raise ValueError(f"latent size {rank} is above 1024")
        rot = rotary.dims
        self.q = Linear(width, heads * (dim + rot), dtype=dtype)
        self.dkv = NormedLinear(width, rank + rot, rank, eps, dtype) \
            if own_rows else None
        self.uk = Linear(rank, heads * dim, dtype=dtype)
        self.uv = Linear(rank, heads * vdim, dtype=dtype)
        self.o = Linear(heads * vdim, width, dtype=dtype)
        self.ready = False

    def store_spec(self) -> Optional[RowSpec]:
        if self.dkv is None:
            return None
        return RowSpec(LatentShape(**self.sizes).width)

    @torch.no_grad()
    def prepare(self):
        wq, wuk, wuv, wo = (m.weight.data for m in (self.q, self.uk, self.uv, self.o))
        self.shape = sh = LatentShape(**self.sizes, f32=wq.dtype == torch.float32)
        H, width = sh.heads, wq.shape[1]

        w = wq.view(H, sh.dim + sh.rot, width)
        w = torch.cat([F.pad(w[:, : sh.dim], (0, 0, 0, sh.dimp - sh.dim)),
                       F.pad(w[:, sh.dim:], (0, 0, 0, sh.rotp - sh.rot))], 1)
        w = w.reshape(H * sh.dq, width)
        if self.dkv is not None:
            w = torch.cat([w, self.dkv.weight.data])
        w = F.pad(w, (0, 0, 0, -w.shape[0] % 8)).contiguous()
        self.w_in = w
        if sh.dq == sh.dim + sh.rot:
            _share(w, self.q, *([self.dkv] if self.dkv is not None else []))

        rpad = (0, sh.rankp - sh.rank)
        uk = F.pad(wuk.view(H, sh.dim, sh.rank), (*rpad, 0, sh.dimp - sh.dim))
        uv = F.pad(wuv.view(H, sh.vdim, sh.rank), (*rpad, 0, sh.vdp - sh.vdim))
        self.w_uk = uk.reshape(H * sh.dimp, sh.rankp).contiguous()
        self.w_uv = uv.reshape(H * sh.vdp, sh.rankp).contiguous()
        # absorbed form: [H, dimp, rankp] into the query, [H, rankp, vdp] out
        self.w_absorb = self.w_uk.view(H, sh.dimp, sh.rankp)
        self.w_emit = self.w_uv.view(H, sh.vdp, sh.rankp).transpose(1, 2).contiguous()
        wo = F.pad(wo.view(width, H, sh.vdim), (0, sh.vdp - sh.vdim))
        self.w_o = wo.reshape(width, H * sh.vdp).contiguous()
        self.ready = True

    def forward(self, h: torch.Tensor, batch: RaggedBatch, store: LayerStore,
                tables) -> torch.Tensor:
        """store: the layer's own, or that of the layer it reads."""
        if not self.ready:
            self.prepare()
        sh = self.shape
        H, nq = sh.heads, sh.heads * sh.dq
        y = ops.linear(h, self.w_in)
        q = y[:, :nq]
        dkv = norm_w = None
        if self.dkv is not None:
            dkv = y[:, nq: nq + sh.rank + sh.rot]
            norm_w = self.dkv.norm.weight
        ragged.latent_append(dkv, norm_w, self.eps, store, q, sh, *tables,
                             batch)
        n, n_req, max_len = batch.short_tokens, batch.n_short, batch.max_short
        if not sh.expandable:
            n, n_req, max_len = batch.n_tokens, batch.n_requests, batch.max_len
        parts = []
        if n:
            qn = q[:n].unflatten(1, (H, sh.dq))[..., : sh.dimp]
            q_abs = torch.bmm(qn.transpose(0, 1).contiguous(), self.w_absorb)
            o = ragged.latent_attention_absorbed(q, q_abs, store, sh,
                                                 self.scale, batch, n_req,
                                                 max_len)
            o = torch.bmm(o, self.w_emit)               # [H, n, vdp]
            parts.append(o.transpose(0, 1).reshape(n, H * sh.vdp))
        if n < batch.n_tokens:
            parts.append(ragged.latent_attention_expanded(
                q, store, self.w_uk, self.w_uv, sh, self.scale, batch))
        out = parts[0] if len(parts) == 1 else torch.cat(parts)
        return ops.linear(out, self.w_o)


class GroupedAttention(nn.Module):
    """Causal softmax attention, ``heads`` query heads over ``kv_heads`` cached
    keys and values.

    ``qk_norm``: RMS norms over the whole query and the whole key projection.
    ``head_norm``: every query and key divided by its own root mean square;
    ``head_weights``: and multiplied by a weight per dimension that the heads
    share.
    ``rotary``: positions on queries and keys; ``turn_values``: positions on the
    values as well, undone on each output by its own position.
    ``window``: how many tokens a token sees, up to itself.
    ``sink``: one learned score per head that enters the softmax's denominator
    and nothing else; ``zero_sink``: that score is 0 for every head.
    ``gate``: every head's output times the sigmoid of a number that a
    projection of the input gives.
    ``own_rows``: otherwise the layer has no keys and values of its own and
    attends to the pages of another layer's store.
    ``vmix``: the share of another layer's values in this layer's, where the
    caller passes such values.
    """

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int,
                 vdim: int, scale: float, eps: float, qk_norm: bool = False,
                 sink: bool = False, dtype: torch.dtype = torch.bfloat16, *,
                 head_norm: bool = False, rotary: Optional[Rotary] = None,
                 turn_values: Optional[Rotary] = None,
                 window: Optional[int] = None, zero_sink: bool = False,
                 head_weights: bool = False, gate: bool = False,
                 own_rows: bool = True):
        super().__init__()
        self.shape = sh = GroupedShape(heads, kv_heads, dim, vdim)
        self.scale, self.eps = float(scale), eps
        self.head_norm, self.window = head_norm or head_weights, window
        self.rotary, self.turn_values = rotary, turn_values
        if qk_norm and self.head_norm:
            raise ValueError("queries and keys are normed whole or per head")

        def lin(out_features):
            if not (qk_norm or head_weights):
                return Linear(width, out_features, dtype=dtype)
            normed = dim if head_weights else out_features
            return NormedLinear(width, out_features, normed, eps, dtype)

        self.q, self.k, self.v = lin(heads * dim), None, None
        if own_rows:
            self.k = lin(kv_heads * dim)
            self.v = Linear(width, kv_heads * vdim, dtype=dtype)
        self.g = Linear(width, heads, dtype=dtype) if gate else None
        self.vmix = None
        if (rotary is None and turn_values is None and not self.head_norm
                and own_rows):
            self.vmix = _param(dtype=dtype)
        if zero_sink:
            self.register_buffer("sink", torch.zeros(heads, dtype=dtype),
                                 persistent=False)
        else:
            self.sink = _param(heads, dtype=dtype) if sink else None
        self.o = Linear(heads * vdim, width, dtype=dtype)
        self.w_in = None
        if max(sh.dimp, sh.vdp) > sh.MAX:
            raise ValueError(f"head sizes {dim}/{vdim} are above {sh.MAX}")
        if rotary is not None and (rotary.dims > dim or rotary.dims % 2):
            raise ValueError(f"{rotary.dims} of {dim} dimensions cannot be "
                             f"rotated in pairs")
        if turn_values is not None and (vdim % 2 or turn_values.dims != vdim):
            raise ValueError("values are rotated whole, in pairs")
        if window is not None and window < 1:
            raise ValueError("a window holds at least the token itself")

    def store_spec(self) -> Optional[RowSpec]:
        return None if self.k is None else RowSpec(self.shape.width)

    @property
    def rows(self):
        """The projections whose outputs ``attend`` takes, in this order."""
        return tuple(m for m in (self.q, self.k, self.v, self.g)
                     if m is not None)

    @torch.no_grad()
    def prepare(self):
        if self.w_in is not None:
            return
        w = torch.cat([m.weight.data for m in self.rows])
        # rows of the projection start at whole vectors
        self.w_in = F.pad(w, (0, 0, 0, -w.shape[0] % 8)).contiguous()
        _share(self.w_in, *self.rows)

    def attend(self, y: torch.Tensor, out: torch.Tensor, batch: RaggedBatch,
               store: LayerStore, first: Optional[torch.Tensor] = None,
               turns: Optional[Turns] = None) -> Optional[torch.Tensor]:
        """y [N, q | k | v | gate | ...], what there is of them; writes out [N,
        heads * vdim].  store: the layer's own, or that of the layer it reads.
        first: values [N, kv_heads * vdim] to mix in.  turns: the tables of
        this layer's rotations.  Returns this layer's values before mixing, a
        view of y."""
        sh, own = self.shape, self.k is not None
        norms = [getattr(m, "norm", None) for m in (self.q, self.k)]
        q = ragged.grouped_append(
            y, *(None if n is None else n.weight for n in norms), self.eps,
            None if first is None else self.vmix, first, store, sh, batch,
            turns, self.head_norm, own)
        values = (sh.heads + sh.kv_heads) * sh.dim
        end = values + sh.kv_heads * sh.vdim if own else sh.heads * sh.dim
        gate = None if self.g is None else y[:, end: end + sh.heads]
        ragged.grouped_attention(q, self.sink, store, sh, self.scale, batch, out,
                                 self.window, turns, gate)
        return y[:, values: end] if own else None

    def forward(self, h: torch.Tensor, batch: RaggedBatch, store: LayerStore,
                first: Optional[torch.Tensor] = None,
                turns: Optional[Turns] = None):
        """Returns (output, values before mixing)."""
        if self.w_in is None:
            self.prepare()
        y = ops.linear(h, self.w_in)
        out = y.new_empty(y.shape[0], self.o.in_features)
        v = self.attend(y, out, batch, store, first, turns)
        return self.o(out), v


class SelectiveScan(nn.Module):
    """Mamba: a diagonal linear recurrence per channel with ``states`` fp32
    states, whose step size, input and read-out vectors depend on the token,
    behind a short convolution and before a silu gate."""

    def __init__(self, width: int, channels: int, states: int, rank: int,
                 taps: int, dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        self.shape = sh = ScanShape(channels, states, rank)
        if states > sh.MAX:
            raise ValueError(f"{states} states are above {sh.MAX}")
        self.add_module("in", Linear(width, 2 * channels, dtype=dtype))
        self.conv = CausalConv(channels, taps, True, dtype)
        self.x = Linear(channels, rank + 2 * states, dtype=dtype)
        self.dt = _Biased(channels, rank, dtype=dtype)
        self.A_log = _param(channels, states, dtype=dtype)
        self.D = _param(channels, dtype=dtype)
        self.o = Linear(channels, width, dtype=dtype)
        self.ready = False

    def store_spec(self) -> LayerSpec:
        sh = self.shape
        return LayerSpec(StateSpec(1, sh.statesp, sh.channels),
                         {"conv": self.conv.history()})

    @torch.no_grad()
    def prepare(self):
        sh, w = self.shape, self.x.weight.data
        # [step input | B | C], each from a whole vector on, zeros between
        self.w_x = w.new_zeros(sh.width, w.shape[1])
        for at, part in zip(sh.columns, w.split([sh.rank, sh.states, sh.states])):
            self.w_x[at: at + part.shape[0]] = part
        self.A = F.pad(-torch.exp(self.A_log.data.float()).T,
                       (0, 0, 0, sh.statesp - sh.states)).contiguous()
        self.D32, self.b32 = self.D.data.float(), self.dt.b.data.float()
        self.ready = True

    def forward(self, h: torch.Tensor, batch: RaggedBatch,
                store: LayerStore) -> torch.Tensor:
        if not self.ready:
            self.prepare()
        sh = self.shape
        x, z = getattr(self, "in")(h).split(sh.channels, 1)
        x = recurrent.causal_conv(x, self.conv.by_tap, self.conv.b,
                                  store.histories["conv"], batch, silu=True)
        y = ops.linear(x, self.w_x)
        dt = ops.linear(y[:, : sh.rank], self.dt.weight)
        return self.o(recurrent.selective_scan(x, z, dt, self.b32, y, self.A,
                                               self.D32, store.state, sh, batch))


class GatedDelta(nn.Module):
    """Gated delta rule: a linear recurrence with a fp32 matrix state per head
    that forgets and corrects (delta write), behind short convolutions, with a
    normed and gated output.

    The decay is one number per head (projection ``a``) and the gate a
    projection ``g``.  ``ranks``: the decay is one number per head and key
    channel, and both come through low-rank projections, ``a2`` of ``a1`` and
    ``g2`` of ``g1``.  ``gate``: silu or sigmoid."""

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int,
                 vdim: int, taps: int, eps: float,
                 dtype: torch.dtype = torch.bfloat16, *,
                 ranks: Optional[Tuple[int, int]] = None, gate: str = "silu"):
        super().__init__()
        if heads % kv_heads:
            raise ValueError(f"{heads} heads do not share {kv_heads} query/key "
                             f"heads evenly")
        if gate not in ("silu", "sigmoid"):
            raise ValueError(f"unknown gate {gate!r}")
        self.shape = DeltaShape(heads, kv_heads, dim, vdim, taps, ranks)
        self.eps, self.sigmoid = eps, gate == "sigmoid"
        lin = lambda i, o: Linear(i, o, dtype=dtype)  # noqa: E731
        self.q = ConvLinear(width, kv_heads * dim, taps, dtype)
        self.k = ConvLinear(width, kv_heads * dim, taps, dtype)
        self.v = ConvLinear(width, heads * vdim, taps, dtype)
        if ranks is None:
            self.g, self.a = lin(width, heads * vdim), lin(width, heads)
        else:
            self.a1, self.a2 = lin(width, ranks[0]), lin(ranks[0], heads * dim)
            self.g1, self.g2 = lin(width, ranks[1]), lin(ranks[1], heads * vdim)
        self.b = lin(width, heads)
        self.A_log = _param(heads, dtype=dtype)
        self.dt_bias = _param(heads * (1 if ranks is None else dim), dtype=dtype)
        self.norm = RMSNorm(vdim, eps, dtype=dtype)
        self.o = lin(heads * vdim, width)
        self.ready = False

    def store_spec(self) -> StateSpec:
        sh = self.shape
        return StateSpec(sh.heads, sh.dim, sh.vdim, sh.channels, sh.taps - 1)

    @torch.no_grad()
    def prepare(self):
        sh, convs = self.shape, (self.q, self.k, self.v)
        self.w_conv = torch.cat([m.conv.weight.data for m in convs]).contiguous()
        if sh.ranks is None:
            rows = (*convs, self.g, self.a, self.b)
            self.w_in = torch.cat([m.weight.data for m in rows]).contiguous()
            _share(self.w_in, *rows)
        else:
            rows = (*convs, self.a1, self.g1, self.b)
            w = self.q.weight.data
            self.w_in = w.new_zeros(-(-(sh.columns[5] + sh.heads) // 8) * 8,
                                    w.shape[1])
            for at, m in zip(sh.columns, rows):
                self.w_in[at: at + m.out_features] = m.weight.data
                m.weight.data = self.w_in[at: at + m.out_features]
            # both second projections in one product, zeros where they do not
            # read
            lo, hi = sh.inputs
            mid, cut = sh.columns[4] - lo, self.a2.out_features
            self.w_low = w.new_zeros(cut + self.g2.out_features, hi - lo)
            for m, part in ((self.a2, self.w_low[:cut, :mid]),
                            (self.g2, self.w_low[cut:, mid:])):
                part = part[:, : m.in_features]
                part.copy_(m.weight.data)
                m.weight.data = part
        self.ready = True

    def forward(self, h: torch.Tensor, batch: RaggedBatch,
                store: LayerStore) -> torch.Tensor:
        if not self.ready:
            self.prepare()
        y, z = ops.linear(h, self.w_in), None
        if self.shape.ranks is not None:
            lo, hi = self.shape.inputs
            z = ops.linear(y[:, lo: hi], self.w_low)
        o = ragged.gated_delta(y, self.w_conv, self.A_log, self.dt_bias,
                               self.norm.weight, store, self.shape, self.eps,
                               batch, z, self.sigmoid)
        return self.o(o)


class GatedMLP(nn.Module):
    """W_down (act(W_gate h) * W_up h)."""

    ACTS = {"gelu_tanh": ops.geglu, "silu": ops.swiglu}

    def __init__(self, width: int, ff: int, act: str,
                 dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        self.act = self.ACTS[act]
        self.gate = Linear(width, ff, dtype=dtype)
        self.up = Linear(width, ff, dtype=dtype)
        self.down = Linear(ff, width, dtype=dtype)
        self.fused = None

    def prepare(self):
        from .fuse import FusedColumns
        self.fused = FusedColumns([self.gate, self.up])

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        g, u = self.fused(h) if self.fused is not None else (self.gate(h), self.up(h))
        return self.down(self.act(g, u))


class BiasedMLP(nn.Module):
    """W_down glu(W_gate h + b, W_up h + b) + b.  The products are plain ones;
    the unit adds its biases itself, and the last one is left to what comes
    next."""

    def __init__(self, width: int, ff: int, glu: ClampedGLU,
                 dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        self.glu = glu
        self.gate = Linear(width, ff, bias=True, dtype=dtype)
        self.up = Linear(width, ff, bias=True, dtype=dtype)
        self.down = Linear(ff, width, bias=True, dtype=dtype)
        self.w_in = None

    @torch.no_grad()
    def prepare(self):
        # both halves of a row begin at whole vectors
        ff = self.gate.out_features
        self.half = -(-ff // 8) * 8
        w = self.gate.weight.data
        self.w_in = w.new_zeros(2 * self.half, w.shape[1])
        for at, m in ((0, self.gate), (self.half, self.up)):
            part = self.w_in[at: at + ff]
            part.copy_(m.weight.data)
            m.weight.data = part

    def rows(self, h: torch.Tensor):
        """(output without the last bias, that bias)."""
        if self.w_in is None:
            self.prepare()
        y, ff = ops.linear(h, self.w_in), self.gate.out_features
        u = self.glu(y[:, :ff], y[:, self.half: self.half + ff],
                     self.gate.bias, self.up.bias)
        return ops.linear(u, self.down.weight), self.down.bias

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        y, bias = self.rows(h)
        return y + bias


class MLP(nn.Module):
    """W_down act(W_up h)."""

    ACTS = {"gelu": ragged.gelu}

    def __init__(self, width: int, ff: int, act: str,
                 dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        self.act = self.ACTS[act]
        self.up = Linear(width, ff, dtype=dtype)
        self.down = Linear(ff, width, dtype=dtype)

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        return self.down(self.act(self.up(h)))


class ParallelBlock(nn.Module):
    """A mixer and a feed-forward (or none) that read the same rows, and the
    sum of what they make of them: one GEMM into both, each writes its part of
    one activation row, one GEMM out of both, whose accumulator holds the sum.
    """

    def __init__(self, mix: nn.Module, mlp: Optional[MLP]):
        super().__init__()
        self.mix, self.mlp = mix, mlp
        self.w_in = self.w_out = None

    @torch.no_grad()
    def prepare(self):
        rows, o = list(self.mix.rows), self.mix.o
        self.mixed = o.in_features              # columns the mixer writes
        self.taken = sum(m.out_features for m in rows)   # ... and reads
        if self.mlp is None:
            self.w_in = torch.cat([m.weight.data for m in rows])
            self.w_out = o.weight.data
        else:
            up, down = self.mlp.up, self.mlp.down
            # units with zero weights round the activation row up
            extra = -(self.mixed + up.out_features) % 8
            rows.append(up)
            self.w_in = F.pad(torch.cat([m.weight.data for m in rows]),
                              (0, 0, 0, extra))
            self.w_out = F.pad(torch.cat([o.weight.data, down.weight.data], 1),
                               (0, extra))
            o.weight.data = self.w_out[:, : self.mixed]
            down.weight.data = self.w_out[:, self.mixed: self.mixed
                                          + down.in_features]
        self.hidden = self.w_out.shape[1] - self.mixed
        # rows of the projection start at whole vectors
        self.w_in = F.pad(self.w_in, (0, 0, 0, -self.w_in.shape[0] % 8))
        self.w_in = self.w_in.contiguous()
        _share(self.w_in, *rows)
        self.mix.w_in = self.w_in[: self.taken]

    def forward(self, h: torch.Tensor, batch: RaggedBatch, store: LayerStore,
                *extra):
        """Returns (sum of both sublayers, what the mixer returns besides)."""
        if self.w_in is None:
            self.prepare()
        y = ops.linear(h, self.w_in)
        z = y.new_empty(y.shape[0], self.w_out.shape[1])
        got = self.mix.attend(y, z[:, : self.mixed], batch, store, *extra)
        if self.mlp is not None:
            self.mlp.act(y[:, self.taken: self.taken + self.hidden],
                         z[:, self.mixed:])
        return ops.linear(z, self.w_out), got


class _Stacked(nn.Module):
    """One matrix per expert, ``weight`` [experts, out, in]."""

    def __init__(self, n: int, out_features: int, in_features: int,
                 dtype: torch.dtype):
        super().__init__()
        self.weight = _param(n, out_features, in_features, dtype=dtype)

    def pad(self, rows: int, cols: int) -> torch.Tensor:
        """The weights with zeros up to this size; the parameter stays a view."""
        n, r, c = self.weight.shape
        w = F.pad(self.weight.data, (0, cols - c, 0, rows - r)).contiguous()
        self.weight.data = w[:, :r, :c]
        return w


class RoutedExperts(nn.Module):
    """Every token's ``top`` of ``experts`` feed-forwards and ``identity``
    experts that return their input.  A feed-forward is ungated with relu^2,
    or gated with ``glu``.  ``routing``: what the router's 32-bit logits become;
    ``correction`` biases the choice but not the weights."""

    def __init__(self, width: int, ff: int, experts: int, identity: int,
                 top: int, dtype: torch.dtype = torch.bfloat16, *,
                 glu: Optional[ClampedGLU] = None, routing: Routing = Routing(),
                 correction: bool = True):
        super().__init__()
        self.shape = sh = ExpertShape(width, ff, experts, identity, top)
        self.glu, self.routing = glu, routing
        if glu is not None:
            self.gate = _Stacked(experts, ff, width, dtype)
        self.up = _Stacked(experts, ff, width, dtype)
        self.down = _Stacked(experts, width, ff, dtype)
        self.router = Linear(width, sh.total, dtype=dtype)
        self.correction = _param(sh.total, dtype=dtype) if correction else None
        self.ready = False

    @torch.no_grad()
    def prepare(self):
        sh = self.shape
        if self.glu is None:
            self.w_up = self.up.pad(sh.ffp, sh.widthp)
        else:  # the gate's rows, then the up projection's
            w = self.up.weight.data
            self.w_up = w.new_zeros(w.shape[0], 2 * sh.ffp, sh.widthp)
            for at, m in ((0, self.gate), (sh.ffp, self.up)):
                part = self.w_up[:, at: at + sh.ff, : sh.width]
                part.copy_(m.weight.data)
                m.weight.data = part
        self.w_down = self.down.pad(sh.width, sh.ffp)
        self.w_router = experts.pack(self.router.weight.data, sh.widthp)
        self.ready = True

    def rows(self, h: torch.Tensor):
        """What a token's experts give, to be summed per token: (rows, where
        [N, top]); h [N, width padded to a multiple of ``ExpertShape.STEP``]."""
        if not self.ready:
            self.prepare()
        if self.shape.identity or not self.routing.on_input:
            raise ValueError("these experts' rows still need their weights")
        return experts.expert_rows(h, self.w_router, self.correction, self.w_up,
                                   self.w_down, self.shape, self.routing,
                                   self.glu)[:2]

    def forward(self, x: torch.Tensor, h: torch.Tensor,
                copy: bool = False) -> Optional[torch.Tensor]:
        """Adds to the residual x in place; h as above.  copy: returns the new
        x in h's type."""
        if not self.ready:
            self.prepare()
        return experts.add_experts(x, h, self.w_router, self.correction,
                                   self.w_up, self.w_down, self.shape, copy,
                                   self.routing, self.glu)


class TokenInput(nn.Module):
    """What a layer takes from a token's own row of an embedding table:
    W_proj (gelu_tanh(W_gate x) * e), to be RMS-normed with ``norm`` and added
    to the residual x."""

    def __init__(self, width: int, dim: int, eps: float,
                 dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        self.gate = Linear(width, dim, dtype=dtype)
        self.proj = Linear(dim, width, dtype=dtype)
        self.norm = RMSNorm(width, eps, dtype=dtype)
        self.w_gate = None

    @torch.no_grad()
    def prepare(self):
        if self.gate.in_features % ExpertShape.STEP == 0:
            self.w_gate = experts.pack(self.gate.weight.data,
                                       self.gate.in_features)

    def forward(self, x: torch.Tensor, e: torch.Tensor,
                copy: Optional[torch.Tensor] = None) -> torch.Tensor:
        """x: fp32 residual; e [N, dim]; copy: x in the weights' type, where
        the caller has it."""
        if (self.w_gate is not None and x.is_cuda
                and x.shape[0] <= experts.FEW):
            g = experts.token_gate(x, self.w_gate, e)
        else:
            g = ops.geglu(self.gate(x.to(e.dtype) if copy is None else copy), e)
        return self.proj(g)
