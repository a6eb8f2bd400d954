"""Sadosun against the plain oracle: mechanisms alone, then the batch engine."""

import math

import pytest
import torch

import sadosun_cases as cases
import sadosun_oracle as oracle
from mlx_sharding_amd.models.mixers import RoutedExperts, TokenInput
from mlx_sharding_amd.ops import experts, ragged, recurrent
from mlx_sharding_amd.ops.experts import ExpertShape
from mlx_sharding_amd.ops.paged import (SPAN, HistorySpec, LayerSpec, LayerStore,
                                        PagedState, RaggedBatch, RowSpec,
                                        StateSpec)
from mlx_sharding_amd.ops.ragged import GroupedShape, Rotary, Turns
from mlx_sharding_amd.ops.recurrent import ScanShape
from mlx_sharding_amd.parallel.batching import BatchEngine


@pytest.fixture(autouse=True)
def one_thread():
    """Tiny tensors: threads only cost."""
    n = torch.get_num_threads()
    torch.set_num_threads(1)
    yield
    torch.set_num_threads(n)


GPU = pytest.param("cuda", marks=pytest.mark.gpu)
DEVICES = ["cpu", GPU]
F32, BF16 = torch.float32, torch.bfloat16
DTYPES = [F32, BF16]


class Feed:
    """Streams of rows through one layer's store, in batches of portions.
    Slots are poisoned, and each stream's result comes back whole."""

    def __init__(self, spec, lens, device, dtype):
        self.state = PagedState([spec], sum(lens.values()) + 64 * len(lens),
                                len(lens) + 1, dtype, device)
        cases.poison(self.state)
        self.store = self.state.layers[0]
        self.state.admit("other")      # so that slots and pages are not the first
        self.state.reserve("other", 1)
        self.lens, self.device, self.dtype = lens, device, dtype

    def run(self, streams, schedule, step):
        """streams {id: tensor [T, ...] or tuple of them}; step(batch, rows...)
        returns rows."""
        at, got = {r: 0 for r in streams}, {r: [] for r in streams}
        for portions in schedule:
            for r, n in portions:
                if r not in self.state.live:
                    self.state.admit(r)
                self.state.reserve(r, at[r] + n)
            live = [(self.state.live[r], n) for r, n in portions]
            batch = RaggedBatch(live, self.device)
            order = [portions[j] for j in batch.order]
            parts = [tuple(x[at[r]: at[r] + n] for x in _tuple(streams[r]))
                     for r, n in order]
            rows = [torch.cat(c).to(self.device) for c in zip(*parts)]
            out = step(batch, *rows).cpu()
            off = 0
            for r, n in order:
                got[r].append(out[off: off + n])
                off += n
                at[r] += n
                self.state.live[r].length = at[r]
        for r in streams:
            self.state.release(r)
        return {r: torch.cat(v) for r, v in got.items()}


def _tuple(x):
    return x if isinstance(x, tuple) else (x,)


LENS = {"a": 150, "b": 20, "c": 67}
SCHEDULE = [[("a", 150), ("b", 20), ("c", 67)]], [
    [("a", 1), ("b", 17), ("c", 2)], [("c", 1), ("a", 64)], [("b", 1), ("a", 2)],
    [("a", 17), ("c", 63), ("b", 2)], [("a", 16)], [("a", 49), ("c", 1)], [("a", 1)]], [
    [(r, 1) for r in LENS if t < LENS[r]] for t in range(150)]


# ---------------------------------------------------------------------------
# Mechanisms alone
# ---------------------------------------------------------------------------

def test_oracle_forms_agree():
    """The row form of the oracle's attention is the token form."""
    g = torch.Generator().manual_seed(0)
    q, k, v = (torch.randn(11, n, 5, generator=g).double() for n in (6, 2, 2))
    for window in (1, 3, 11, 50):
        assert torch.allclose(oracle.attend(q, k, v, 0.7, window),
                              oracle.attend_rows(q, k, v, 0.7, window))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("C,taps", [(40, 3), (17, 4), (64, 1), (24, 8), (9, 2)])
def test_causal_conv(device, dtype, C, taps):
    g = torch.Generator().manual_seed(1)
    w = (torch.randn(C, taps, generator=g)).to(dtype)
    b = torch.randn(C, generator=g).to(dtype)
    streams = {r: torch.randn(n, C + 5, generator=g).to(dtype) for r, n in LENS.items()}
    on = lambda t: t.to(device)  # noqa: E731
    tol = 1e-6 if dtype == F32 else 1e-2
    for bias, add, silu, pad in ((b, False, True, 1), (None, True, False, 16)):
        feed = Feed(LayerSpec(None, {"h": HistorySpec(C, taps - 1)}), LENS, device, dtype)

        def step(batch, rows):
            out = recurrent.causal_conv(
                rows[:, :C], on(w.T.contiguous()), None if bias is None else on(bias),
                feed.store.histories["h"], batch, add, silu, pad)
            assert out.shape[1] % pad == 0 and bool((out[:, C:] == 0).all())
            return out[:, :C]
        for schedule in SCHEDULE:
            got = feed.run(streams, schedule, step)
            for r, x in streams.items():
                h = x[:, :C].double()
                y = oracle.causal_conv(h, w.double())
                if bias is not None:
                    y = y + bias.double()
                if silu:
                    y = oracle.silu(y)
                assert cases.error(got[r], y + h if add else y) < tol


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W,taps", [(40, 3), (97, 4), (1024, 2), (2500, 5),
                                    (4100, 8), (9000, 4), (64, 1)])
def test_norm_conv(device, dtype, W, taps):
    """Residual update, norm with one number, convolution of the normed rows."""
    g = torch.Generator().manual_seed(2)
    eps = 0.05  # large, so that a misplaced eps shows
    one = torch.tensor(1.3).to(dtype)
    post = (1 + 0.3 * torch.randn(W, generator=g)).to(dtype)
    w = torch.randn(W, taps, generator=g).to(dtype)
    lens = {"a": 40, "b": 19}
    streams = {r: (torch.randn(n, W, generator=g), (3 * torch.randn(n, W, generator=g)).to(dtype))
               for r, n in lens.items()}
    schedules = [[("a", 40), ("b", 19)]], [[("a", 1), ("b", 17)], [("b", 2), ("a", 3)],
                                           [("a", 20)], [("a", 16)]]
    tol = 1e-6 if dtype == F32 else 8e-3
    for use_y, use_post in ((False, False), (True, False), (True, True)):
        feed = Feed(LayerSpec(None, {"h": HistorySpec(W, taps - 1)}), lens, device, dtype)
        on = lambda t: t.to(device)  # noqa: E731

        def step(batch, x, y):
            x = x.clone()
            out = recurrent.norm_conv(x, y if use_y else None, on(post) if use_post else None,
                                      on(one), eps, on(w.T.contiguous()),
                                      feed.store.histories["h"], batch, dtype, 64)
            assert out.shape[1] % 64 == 0 and bool((out[:, W:] == 0).all())
            return torch.cat([out[:, :W].float(), x], 1)
        for schedule in schedules:
            got = feed.run(streams, schedule, step)
            for r, (x, y) in streams.items():
                want = x.double()
                if use_y:
                    y = y.double()
                    want = want + (oracle.rms(y, eps) * post.double() if use_post else y)
                h = oracle.rms(want, eps) * one.double()
                assert cases.error(got[r][:, W:], want) < 1e-6
                assert cases.error(got[r][:, :W], oracle.with_recent(h, w.double())) < tol


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("C,N", [(70, 16), (256, 1), (33, 12), (8, 70), (20, 300), (64, 32)])
def test_scan(device, dtype, C, N):
    """From states that forget at once to ones that hardly forget; over many
    spans, in portions, beside others."""
    sh = ScanShape(C, N, 5)
    g = torch.Generator().manual_seed(3)
    lens = {"a": 3 * SPAN + 7, "b": SPAN, "c": 30, "d": SPAN + 1}
    A = -torch.exp(torch.linspace(-6, 2, N).expand(C, N) + 0.3 * torch.randn(C, N, generator=g))
    D, bias = torch.randn(C, generator=g), torch.linspace(-9, 3, C)
    Ap = torch.nn.functional.pad(A.T, (0, 0, 0, sh.statesp - N)).contiguous()

    def bc_row(n):
        out = torch.zeros(n, sh.width)
        for at in sh.columns[1:]:
            out[:, at: at + N] = torch.randn(n, N, generator=g)
        return out.to(dtype)
    streams = {r: (*(torch.randn(n, C, generator=g).to(dtype) for _ in range(3)), bc_row(n))
               for r, n in lens.items()}
    feed = Feed(StateSpec(1, sh.statesp, C), lens, device, dtype)
    on = lambda t: t.to(device)  # noqa: E731

    def step(batch, x, z, dt, bc):
        return recurrent.selective_scan(x, z, dt, on(bias), bc, on(Ap), on(D),
                                        feed.store.state, sh, batch)
    tol = 1e-5 if dtype == F32 else 2e-2
    want = {}
    for r, (x, z, dt, bc) in streams.items():
        x, z, dt, bc = (t.double() for t in (x, z, dt, bc))
        B, Cm = (bc[:, at: at + N] for at in sh.columns[1:])
        y = oracle.scan(x, oracle.softplus(dt + bias.double()), A.double(), B, Cm, D.double())
        want[r] = y * oracle.silu(z)
    for schedule in ([[(r, n) for r, n in lens.items()]],
                     [[("a", 200), ("c", 1), ("b", 17)], [("a", 16), ("b", SPAN - 18), ("d", 2)],
                      [("c", 3), ("d", SPAN - 1), ("b", 1), ("a", lens["a"] - 218)],
                      [("a", 2), ("c", 26)]]):
        got = feed.run(streams, schedule, step)
        for r in lens:
            assert cases.error(got[r], want[r]) < tol, r


@pytest.mark.parametrize("device", DEVICES)
def test_scan_remembers(device):
    """One loud input, read out long after; a state lost at a span's or a
    portion's edge would show."""
    C, N, T, at = 16, 4, 5 * SPAN, SPAN - 3
    sh = ScanShape(C, N, 1)
    A = torch.full((C, N), -1e-4)
    x = torch.zeros(T, C)
    x[at] = 100.0
    bc = torch.zeros(T, sh.width)
    for c in sh.columns[1:]:
        bc[:, c: c + N] = 1.0
    z, dt = torch.full((T, C), 3.0), torch.zeros(T, C)
    feed = Feed(StateSpec(1, sh.statesp, C), {"a": T}, device, F32)
    on = lambda t: t.to(device)  # noqa: E731
    Ap = torch.nn.functional.pad(A.T, (0, 0, 0, sh.statesp - N)).contiguous()

    def step(batch, *rows):
        x, z, dt, bc = rows
        return recurrent.selective_scan(x, z, dt, on(torch.zeros(C)), bc, on(Ap),
                                        on(torch.zeros(C)), feed.store.state, sh, batch)
    B = torch.ones(T, N).double()
    want = oracle.scan(x.double(), oracle.softplus(dt.double()), A.double(), B, B,
                       torch.zeros(C).double()) * oracle.silu(z.double())
    assert float(want[-1].min()) > 100 and float(want[at - 1].abs().max()) == 0
    for sizes in ([T], [at, 1, 2, 300, 1, 17], [at + 1, T], [SPAN], [16]):
        got = feed.run({"a": (x, z, dt, bc)}, [[("a", n)] for n in cases.cut(T, sizes)], step)
        assert cases.error(got["a"], want) < 1e-5, sizes


SHAPES = {
    "usual": ExpertShape(96, 80, 12, 4, 4),
    "no identity": ExpertShape(64, 64, 8, 0, 2),
    "odd": ExpertShape(51, 33, 5, 2, 3),
    "all": ExpertShape(40, 8, 3, 2, 5),
    "one": ExpertShape(17, 1, 1, 0, 1),
    "many": ExpertShape(128, 24, 190, 40, 9),
    "most identity": ExpertShape(72, 130, 2, 30, 6),
    "more picks than lanes": ExpertShape(32, 8, 60, 40, 70),
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", SHAPES)
@pytest.mark.parametrize("n", [1, 15, 70, 400])
def test_experts(device, dtype, kind, n):
    """Few and many tokens per expert; x moves by the weighted sum."""
    sh = SHAPES[kind]
    g = torch.Generator().manual_seed(n)
    m = RoutedExperts(sh.width, sh.ff, sh.experts, sh.identity, sh.top, dtype)
    for t, gain in ((m.up.weight, sh.width ** -0.5), (m.down.weight, sh.ff ** -0.5),
                    (m.router.weight, 2 * sh.width ** -0.5), (m.correction, 0.1)):
        t.data = (torch.randn(t.shape, generator=g) * gain).to(dtype)
    w = {"m.router": m.router.weight.double(), "m.correction": m.correction.double()}
    for e in range(sh.experts):
        w[f"m.e{e}.up"] = m.up.weight[e].double()
        w[f"m.e{e}.down"] = m.down.weight[e].double()
    h = torch.randn(n, sh.width, generator=g).to(dtype)
    x = torch.randn(n, sh.width, generator=g)
    want = x.double() + oracle.experts(h.double(), w, "m.", cases.moe(
        sh.ff, sh.experts, sh.top, sh.identity))
    m.to(device)
    xd = x.to(device)
    hp = torch.nn.functional.pad(h, (0, sh.widthp - sh.width)).to(device)
    copy = m(xd, hp, copy=True)
    assert cases.error(xd, want) < (5e-6 if dtype == F32 else 2e-2)
    assert copy.dtype == dtype and torch.equal(copy, xd.to(dtype))
    x2 = x.to(device)
    assert m(x2, hp) is None and torch.equal(x2, xd)


def test_operand_layout():
    w = torch.arange(23 * 70).float().view(23, 70)
    p = experts.pack(w, 128)
    assert p.shape == (2, 4, 64, 8)
    e, c = 21, 61
    assert float(p[e // 16, c // 32, c // 8 % 4 * 16 + e % 16, c % 8]) == float(w[e, c])
    assert torch.equal(experts.unpack(p, 23, 70), w)


@pytest.mark.gpu
@pytest.mark.parametrize("tile", [16, 128])
def test_tile_sizes_agree(tile, monkeypatch):
    """Both grouped products on the same few and many tokens."""
    monkeypatch.setattr(ExpertShape, "tile", lambda self, tokens: tile)
    for kind in ("usual", "odd", "many"):
        for n in (3, 130):
            test_experts("cuda", BF16, kind, n)
            test_experts("cuda", F32, kind, n)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_correction_biases_the_choice_only(device, dtype):
    """A correction that forces a poor expert: it is chosen, with the weight of
    its own score."""
    sh = ExpertShape(32, 16, 4, 2, 2)
    g = torch.Generator().manual_seed(0)
    router = torch.randn(6, 32, generator=g).to(dtype)
    corr = torch.tensor([0.0, 0.0, 50.0, 0.0, 0.0, 7.0]).to(dtype)
    up = torch.randn(4, 16, 32, generator=g).to(dtype)
    down = torch.randn(4, 32, 16, generator=g).to(dtype)
    h = torch.randn(20, 32, generator=g).to(dtype)
    z = h.double() @ router.double().T
    s = torch.softmax(z, -1)
    a, b = s[:, 2:3], s[:, 5:]
    y2 = torch.clamp(h.double() @ up[2].double().T, min=0) ** 2 @ down[2].double().T
    want = (a * y2 + b * h.double()) / (a + b + 1e-20)
    pad = torch.nn.functional.pad
    x = torch.zeros(20, 32, device=device)
    experts.add_experts(x, pad(h, (0, 32)).to(device),
                        experts.pack(router, 64).to(device),
                        corr.to(device), pad(up, (0, 32, 0, 48)).to(device),
                        pad(down, (0, 48)).to(device), sh)
    assert cases.error(x, want) < (1e-5 if dtype == F32 else 2e-2)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W,dim", [(64, 24), (51, 5), (128, 1), (256, 64)])
@pytest.mark.parametrize("n", [1, 30, 90])
def test_token_input(device, dtype, W, dim, n):
    g = torch.Generator().manual_seed(4)
    m = TokenInput(W, dim, 1e-2, dtype)
    m.gate.weight.data = (torch.randn(dim, W, generator=g) * W ** -0.5).to(dtype)
    m.proj.weight.data = (torch.randn(W, dim, generator=g) * dim ** -0.5).to(dtype)
    m.norm.weight.data = (1 + 0.3 * torch.randn(W, generator=g)).to(dtype)
    x = torch.randn(n, W, generator=g).to(dtype).float()
    table = torch.randn(n, 3 * dim, generator=g).to(dtype)
    w = {"s." + k.replace(".weight", ""): v.double() for k, v in m.state_dict().items()}
    e = table[:, dim: 2 * dim]
    want = x.double() + oracle.token_input(x.double(), e.double(), w, "s.", 1e-2)
    m.to(device).prepare()
    xd, td = x.to(device), table.to(device)
    for copy in (None, xd.to(dtype)):
        y = m(xd, td[:, dim: 2 * dim], copy)
        x2 = xd.clone()
        ragged.add_norm(x2, y, m.norm.weight, None, 1e-2, 0.0, dtype)
        assert cases.error(x2, want) < (2e-6 if dtype == F32 else 2e-2)


def batch_of(portions, device, max_tokens=640):
    """Requests {id: (held, new)} and their batch."""
    state = PagedState([], max_tokens, 8, F32, device)
    for r, (p, n) in portions.items():
        state.admit(r)
        state.reserve(r, p + n)
        state.live[r].length = p
    return state, RaggedBatch([(state.live[r], n) for r, (_, n) in portions.items()], device)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,V,rot", [(6, 2, 24, 40, 16), (2, 1, 18, 6, 2), (4, 4, 128, 64, 128),
                                         (3, 3, 272, 8, 200), (8, 2, 64, 32, 64), (1, 1, 2, 2, 2)])
def test_append(device, dtype, H, G, D, V, rot):
    """Queries and keys rotated and normed per head, values rotated; each in
    its slot, and slots before a portion's start keep what they hold."""
    portions = {"a": (60, 1), "b": (3, 70), "c": (0, 16), "d": (130, 17), "e": (64, 64)}
    state, batch = batch_of(portions, device)
    sh = GroupedShape(H, G, D, V)
    g = torch.Generator().manual_seed(5)
    store = LayerStore(RowSpec(sh.width), state.n_pages, 1, dtype, device)
    store.rows.fill_(float("nan"))
    N, base, eps = batch.n_tokens, 100.0, 0.3
    y = (torch.randn(N, (H + G) * D + G * V + 3, generator=g) * 2).to(dtype)
    y = torch.nn.functional.pad(y, (0, -y.shape[1] % 8))
    q, k, v = (t.reshape(N, n, -1) for t, n in zip(
        y.double()[:, : (H + G) * D + G * V].split([H * D, G * D, G * V], 1), (H, G, G)))
    pos = batch.tok_pos.cpu()
    tol = 2e-6 if dtype == F32 else 8e-3
    tables = lambda n: Rotary(n, base).tables(1024, device)  # noqa: E731
    for turns, norm in ((Turns(tables(rot), tables(V)), True), (Turns(tables(rot)), False),
                        (None, True), (Turns(None, tables(V)), True)):
        wq, wk, wv = q, k, v
        if turns is not None and turns.qk is not None:
            wq, wk = (oracle.turn(t, pos, base, rot) for t in (wq, wk))
        if norm:
            wq, wk = oracle.rms(wq, eps), oracle.rms(wk, eps)
        if turns is not None and turns.v is not None:
            wv = oracle.turn(wv, pos, base, V)
        got = ragged.grouped_append(y.to(device), None, None, eps, None, None, store, sh,
                                    batch, turns, norm)
        assert got.shape == (N, H, sh.dimp) and bool((got[..., D:] == 0).all())
        assert cases.error(got[..., :D].reshape(N, -1), wq.reshape(N, -1)) < tol
        for t0, n, p0, held in batch.host:
            pages = torch.tensor(held.pages, device=device)
            kk = sh.keys(store.rows)[pages].reshape(-1, G, sh.dimp)
            vv = sh.values(store.rows)[pages].reshape(-1, G, sh.vdp)
            assert bool(torch.isnan(kk[:p0]).all()) and bool(torch.isnan(vv[:p0]).all())
            kk, vv = kk[p0: p0 + n], vv[p0: p0 + n]
            assert bool((kk[..., D:] == 0).all()) and bool((vv[..., V:] == 0).all())
            at = slice(t0, t0 + n)
            assert cases.error(kk[..., :D].reshape(n, -1), wk[at].reshape(n, -1)) < tol
            assert cases.error(vv[..., :V].reshape(n, -1), wv[at].reshape(n, -1)) < tol


class Mixer:
    """The mixer of one layer with its storage: feed portions, compare."""

    def __init__(self, layer, width, dtype, device, w=None, seed=0, eps=1e-5):
        cfg = cases.config(width, 8, [layer], eps)
        self.w = w or cases.weights(cfg, seed)
        self.model = cases.build(cfg, self.w, device, dtype)
        self.layer, self.dtype, self.device, self.eps = layer, dtype, device, eps

    def want(self, h, w=None, **changes):
        w = {k: v.double() for k, v in (w or self.w).items()}
        mx = {**self.layer["mixer"], **changes}
        h = h.to(self.dtype).double()
        if self.layer["type"] == "attention":
            return oracle.attention(h, w, "l0.mix.", mx, self.eps)
        return oracle.mamba(h, w, "l0.mix.", mx)

    def run(self, h, sizes):
        """h [T, width] in portions of these sizes (the last one repeated)."""
        T = h.shape[0]
        state = self.model.make_state(T + 64, 2)
        cases.poison(state)
        state.admit("other")       # so that the pages are not the first
        state.reserve("other", 1)
        held = state.admit("x")
        layer, outs, at = self.model.l0, [], 0
        for n in cases.cut(T, sizes):
            state.reserve("x", at + n)
            batch = RaggedBatch([(held, n)], self.device)
            x = h[at: at + n].to(self.device, self.dtype)
            if self.layer["type"] == "attention":
                y, _ = layer.mix(x, batch, state.layers[0], None,
                                 self.model._turns(layer, batch, batch.cu.device))
            else:
                y = layer.mix(x, batch, state.layers[0])
            outs.append(y.cpu())
            at += n
            held.length = at
        return torch.cat(outs)


LAYERS = {
    "grouped": cases.attention(6, 2, 24, 40, 50, rot=16),
    "one": cases.attention(1, 1, 2, 2, 7),
    "own keys": cases.attention(5, 5, 32, 16, 64),
    "shared keys": cases.attention(20, 1, 16, 24, 100, base=37.0),
    "odd": cases.attention(6, 3, 18, 6, 33, rot=10, scale=2.0),
    "itself": cases.attention(4, 2, 32, 32, 1),
    "pair": cases.attention(4, 2, 32, 32, 2),
    "64/128": cases.attention(4, 2, 64, 128, 65),
    "128": cases.attention(8, 2, 128, 128, 129),
    "256/80": cases.attention(4, 2, 256, 80, 31),
    "all": cases.attention(4, 1, 96, 96, 4096),
    "too wide for prompts": cases.attention(4, 2, 272, 272, 40),
    "widest": cases.attention(2, 1, 512, 512, 90, rot=64),
    "scan": cases.mamba(72, 12, 7, 3),
    "scan, many states": cases.mamba(40, 100, 20, 6),
    "scan, ones": cases.mamba(1, 1, 1, 1),
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", LAYERS)
def test_mixers(device, dtype, kind):
    m = Mixer(LAYERS[kind], 64, dtype, device, eps=0.2)
    h = torch.randn(330, 64, generator=torch.Generator().manual_seed(3))
    tol = 2e-5 if dtype == F32 else 8e-2
    want = m.want(h)
    for sizes in ([330], [1], [64, 17, 2, 60], [16], [2, 3, 129]):
        assert cases.error(m.run(h, sizes), want) < tol, sizes


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_one_in_the_denominator(device, dtype):
    """Scores far below 0 leave almost nothing, scores far above almost all."""
    for scale in (1e-3, 0.3, 3.0):
        m = Mixer(cases.attention(4, 2, 32, 32, 70, scale=scale), 64, dtype, device)
        h = torch.randn(300, 64, generator=torch.Generator().manual_seed(3))
        want = m.want(h)
        w = {k: v.double() for k, v in m.w.items()}
        x = h.to(dtype).double()
        pos = torch.arange(300)
        q, k = (oracle.rms(oracle.turn((x @ w[f"l0.mix.{n}"].T).view(300, -1, 32), pos, 1e4, 32),
                           m.eps) for n in "qk")
        s = (q[0, 0] @ k[0, 0]) * scale     # the first token sees only itself
        v0 = (x @ w["l0.mix.v"].T).view(300, 2, 32)[0, 0]
        p = math.exp(s) / (1 + math.exp(s))
        part = torch.zeros(128).double()
        part[:32] = p * v0
        got = part @ w["l0.mix.o"].T
        if scale == 0.3:
            other = Mixer(cases.attention(1, 1, 32, 32, 70, scale=scale), 64, dtype, device,
                          {**m.w, "l0.mix.q": m.w["l0.mix.q"][:32], "l0.mix.k": m.w["l0.mix.k"][:32],
                           "l0.mix.v": m.w["l0.mix.v"][:32], "l0.mix.o": m.w["l0.mix.o"][:, :32]})
            assert cases.error(other.run(h[:1], [1]), got[None]) < (1e-5 if dtype == F32 else 2e-2)
        # sharp scores carry the rounding of queries and keys
        tol = 1e-5 if dtype == F32 else 2e-2 * max(1.0, 3 * scale)
        for sizes in ([300], [290, 1], [64, 17, 2, 100], [16]):
            assert cases.error(m.run(h, sizes), want) < tol, (scale, sizes)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [64, 130, 200])
def test_window_edges(device, dtype, window):
    """Queries of one head that look for one key: just inside and just outside
    the window, the token itself, the first token, keys at page and tile
    borders.  A seen key carries most of the weight, so a window that is one
    token off cannot hide."""
    layer = cases.attention(4, 2, 32, 24, window, rot=8, base=1e6, scale=0.4)
    m = Mixer(layer, 224, dtype, device, seed=1)
    w = {k: v.double() for k, v in m.w.items()}
    D, T, head = 32, 460, 2
    g = torch.Generator().manual_seed(5)
    h = torch.randn(T, 224, generator=g, dtype=torch.float64)
    asks, last, gone = {}, [], []

    def ask(q, k):
        """Unless one of the two has a part already."""
        taken = {*asks, *asks.values()}
        if 0 <= k < q < T and q not in taken and k not in taken:
            asks[q] = k
            return [q]
        return []
    for q in (window - 1, 255, 256, 319, 383, 400, 449):
        last += ask(q, q - window + 1)      # the last one seen
    for k in (0, 63, 64, 127, 128, 191, 203):
        last += ask(k + window - 1, k)
    for q in (window + 2, 257, 261, 320, 385, 402, 451):
        gone += ask(q, q - window)          # just gone
    for k in (15, 62, 65, 129, 192, 223, 230):
        gone += ask(k + window, k)
    assert len(last) > 5 and len(gone) > 5
    for q, k in ((40, 1), (63, 16), (448, 448 - window // 2), (447, 446)):
        ask(q, k)
    pos = torch.arange(T)
    keys = (h @ w["l0.mix.k"].T).view(T, 2, D)[:, head // 2][:, None]
    keys = oracle.turn(keys, pos, 1e6, 8)
    for q, k in asks.items():
        back = oracle.turn(keys[k: k + 1], pos[q: q + 1], 1e6, 8, -1.0)[0, 0]
        want = torch.randn(4 * D, generator=g, dtype=torch.float64)
        want[head * D: (head + 1) * D] = back
        h[q] = torch.linalg.lstsq(w["l0.mix.q"], want[:, None]).solution[:, 0] * 10
        keys[q] = oracle.turn((w["l0.mix.k"] @ h[q]).view(1, 2, D)[:, head // 2][:, None],
                              pos[q: q + 1], 1e6, 8)[0]
    h = h.to(dtype).double()
    qs, ks = (oracle.rms(oracle.turn((h @ w[f"l0.mix.{n}"].T).view(T, -1, D), pos, 1e6, 8), m.eps)
              for n in "qk")
    for q, k in asks.items():
        lo = max(0, q - window + 1)
        s = torch.exp(ks[lo: q + 1, head // 2] @ qs[q, head] * 0.4)
        if k >= lo:
            assert s[k - lo] / (1 + s.sum()) > 0.5, (q, k)
        else:       # it would have carried the row
            e = torch.exp(ks[k, head // 2] @ qs[q, head] * 0.4)
            assert e / (1 + e + s.sum()) > 0.5, (q, k)
    want = m.want(h)
    rows = sorted(asks)
    for off in (-1, 1):
        other = m.want(h, mask={"size": window + off})
        assert cases.error(other[rows], want[rows]) > 0.3
    tol = 2e-5 if dtype == F32 else 4e-2
    for sizes in ([T], [90, 1], [T - 70, 1], [128, 128, 2], [97, 3], [16], [63, 2, 65]):
        got = m.run(h, sizes)
        assert cases.error(got[rows], want[rows]) < tol, sizes


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_values_turn_with_distance(device, dtype):
    """Each token attends to one key; what it gives depends on how far away
    that is, and not on where the pair lies."""
    layer = cases.attention(2, 1, 16, 16, 300, rot=2, base=50.0)
    m = Mixer(layer, 64, dtype, device)
    h = torch.randn(310, 64, generator=torch.Generator().manual_seed(6))
    want = m.want(h)
    w = {k: v.double() for k, v in m.w.items()}
    x = h.to(dtype).double()
    pos = torch.arange(310)
    q, k = (oracle.rms(oracle.turn((x @ w[f"l0.mix.{n}"].T).view(310, -1, 16), pos, 50.0, 2), m.eps)
            for n in "qk")
    plain = oracle.attend_rows(q, k, (x @ w["l0.mix.v"].T).view(310, 1, 16),
                               layer["mixer"]["scale"], 300)
    assert cases.error(plain.reshape(310, -1) @ w["l0.mix.o"].T, want) > 0.3
    shifted = oracle.turn(oracle.attend_rows(
        q, k, oracle.turn((x @ w["l0.mix.v"].T).view(310, 1, 16), pos + 1000, 50.0, 16),
        layer["mixer"]["scale"], 300), pos + 1000, 50.0, 16, -1.0)
    assert cases.error(shifted.reshape(310, -1) @ w["l0.mix.o"].T, want) < 1e-9
    for sizes in ([310], [1], [200, 3]):
        assert cases.error(m.run(h, sizes), want) < (2e-5 if dtype == F32 else 3e-2)


@pytest.mark.parametrize("device", DEVICES)
def test_future_is_not_seen(device):
    """A loud token at i + 1 does not change what token i gives."""
    for layer in (cases.attention(4, 2, 32, 16, 50), cases.mamba(48, 8, 4, 4)):
        m = Mixer(layer, 64, F32, device)
        h = torch.randn(150, 64, generator=torch.Generator().manual_seed(3))
        base = m.run(h, [150])
        for i in (0, 15, 16, 31, 62, 63, 64, 127, 128):
            loud = h.clone()
            loud[i + 1:] = 50 * torch.randn(149 - i, 64)
            assert torch.equal(m.run(loud, [150])[: i + 1], base[: i + 1]), i


def test_other_combinations():
    """The pieces are usable apart: positions without a window, a window with
    learned sinks and norms over whole rows."""
    from mlx_sharding_amd.models.mixers import GroupedAttention
    m = GroupedAttention(32, 4, 2, 16, 8, 0.25, 1e-5, qk_norm=True, sink=True, dtype=F32, window=9)
    g = torch.Generator().manual_seed(8)
    for p in m.parameters():
        p.data = torch.randn(p.shape, generator=g)
    state = PagedState([m.store_spec()], 64, 1, F32, "cpu")
    held = state.admit(0)
    state.reserve(0, 40)
    h = torch.randn(40, 32, generator=g)
    got, _ = m(h, RaggedBatch([(held, 40)], "cpu"), state.layers[0])
    q = oracle.rms(h @ m.q.weight.T, 1e-5) * m.q.norm.weight
    k = oracle.rms(h @ m.k.weight.T, 1e-5) * m.k.norm.weight
    v = (h @ m.v.weight.T).view(40, 2, 8)
    q, k = q.view(40, 4, 16), k.view(40, 2, 16)
    out = torch.zeros(40, 4, 8)
    for i in range(40):
        for hd in range(4):
            lo = max(0, i - 8)
            e = torch.exp(k[lo: i + 1, hd // 2] @ q[i, hd] * 0.25)
            out[i, hd] = e / (e.sum() + torch.exp(m.sink[hd])) @ v[lo: i + 1, hd // 2]
    assert cases.error(got, out.view(40, -1) @ m.o.weight.T) < 1e-4
    for bad in (dict(window=0), dict(rotary=Rotary(18, 10.0)), dict(rotary=Rotary(3, 10.0)),
                dict(turn_values=Rotary(6, 10.0))):
        with pytest.raises(ValueError):
            GroupedAttention(32, 4, 2, 16, 8, 0.25, 1e-5, **bad)
    for bad in ((8, 8, 2, 1, 4), (8, 8, 1000, 30, 4), (8, 8, 2, 0, 0)):
        with pytest.raises(ValueError):
            ExpertShape(*bad)


# ---------------------------------------------------------------------------
# The engine: whole models, portions, batches, pages and slots
# ---------------------------------------------------------------------------

def engine(name, device, dtype, max_tokens=512, max_requests=4, seed=0):
    cfg = cases.CONFIGS[name]
    e = BatchEngine(cases.build(cfg, cases.weights(cfg, seed), device, dtype),
                    max_tokens, max_requests)
    cases.poison(e.state)
    return e


def test_every_part_shows():
    """The tests' weights make each mechanism visible in the logits."""
    import copy
    cfg, w = cases.CONFIGS["mixed"], cases.weights(cases.CONFIGS["mixed"])
    toks = cases.tokens(cfg, 80)
    want = cases.expected("mixed", toks)

    def off(change=lambda t: None, edit=lambda c: None):
        other, c = {k: v.clone() for k, v in w.items()}, copy.deepcopy(cfg)
        change(other)
        edit(c)
        return cases.error(oracle.forward(c, other, toks), want)

    assert off() == 0
    for i, layer in enumerate(cfg["layers"]):
        names = ["norm1", "canon1", "side.gate", "side.proj", "side.norm"]
        if layer["mlp"] is not None:
            names += ["norm2", "canon2", "mlp.router", "mlp.correction", "mlp.e0.up"]
        if layer["type"] == "mamba1":
            names += ["mix.conv", "mix.conv.b", "mix.dt", "mix.dt.b", "mix.A_log", "mix.D"]
        for n in names:
            def change(t, key=f"l{i}.{n}"):
                t[key] = torch.zeros_like(t[key])
            assert off(change) > 0.005, (i, n)
    for edit in (lambda c: c["embedding"].update(scale=2.0),
                 lambda c: c["norm"].update(eps=0.3),
                 lambda c: c["layers"][0]["mixer"]["mask"].update(size=36),
                 lambda c: c["layers"][0]["mixer"]["rot"].update(dims=14),
                 lambda c: c["layers"][2]["mixer"]["rot"].update(base=250.0),
                 lambda c: c["layers"][2]["mixer"].update(scale=0.2),
                 lambda c: c["layers"][0]["mlp"]["router"].update(top=2)):
        assert off(edit=edit) > 0.005


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", cases.CONFIGS)
def test_portions(device, dtype, name):
    """A prompt whole, token by token, and in portions of many sizes."""
    toks = cases.tokens(cases.CONFIGS[name], 140)
    want = cases.expected(name, toks)
    e = engine(name, device, dtype)
    for sizes in ([140], [1], [2], [3, 16, 17, 1, 1, 64, 38], [65, 63, 12], [128, 2]):
        got = cases.replay(e, {"r": toks}, [[("r", n)] for n in cases.cut(140, sizes)])
        assert cases.model_error(got["r"], want, dtype) < 1, sizes
        assert not e.live and e.state.free_tokens == 512


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_layers(device, dtype, name):
    """The residual stream after every layer."""
    cfg = cases.CONFIGS[name]
    toks = cases.tokens(cfg, 37)
    want = []
    oracle.forward(cfg, cases.weights(cfg), toks, layers_out=want)
    m = cases.build(cfg, cases.weights(cfg), device, dtype)
    state = m.make_state(64, 1)
    held = state.admit(0)
    state.reserve(0, 37)
    got = []
    m.run(torch.tensor(toks, device=device), RaggedBatch([(held, 37)], device),
          state, layer_outputs=got)
    assert len(got) == len(want) == len(cfg["layers"])
    for g, w in zip(got, want):
        assert g.dtype == F32
        assert cases.model_error(g, w, dtype) < 1


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "odd", "wide"])
def test_unequal_batch(device, dtype, name):
    """Portions of prompts beside single tokens; requests pause, end, and
    others take over their pages and slots."""
    cfg = cases.CONFIGS[name]
    lens = {"a": 150, "b": 1, "c": 40, "d": 67, "e": 130, "f": 20}
    streams = {r: cases.tokens(cfg, n, 10 + i) for i, (r, n) in enumerate(lens.items())}
    schedule = [
        [("a", 17), ("b", 1)],
        [("c", 2), ("a", 1), ("d", 66)],
        [("d", 1), ("a", 64), ("c", 16)],           # d ends
        [("e", 64), ("c", 1), ("a", 2)],
        [("c", 1), ("e", 1)],                       # a pauses
        [("a", 17), ("f", 19), ("c", 20), ("e", 2)],  # c ends
        [("f", 1), ("e", 60), ("a", 46)],           # f ends
        [("a", 1), ("e", 1)],
        [("a", 1), ("e", 1)],
        [("e", 1), ("a", 1)],                       # order swaps; both end
    ]
    e = engine(name, device, dtype, max_tokens=448)
    got = cases.replay(e, streams, schedule)
    for r, toks in streams.items():
        n = sum(k for step in schedule for q, k in step if q == r)
        want = cases.expected(name, toks)[:n]
        assert cases.model_error(got[r], want, dtype) < 1, r
    for r in list(e.live):
        e.end(r)
    assert e.state.free_tokens == 448 and e.state.free_slots == 4


@pytest.mark.parametrize("device", DEVICES)
def test_pages_and_slots_are_used_again(device):
    """A pool that just fits runs many requests one after another, and its
    pages and slots in another order each time."""
    e = engine("mixed", device, F32, max_tokens=256, max_requests=2)
    cfg = cases.CONFIGS["mixed"]
    for k in range(4):
        a, b = cases.tokens(cfg, 130, 20 + k), cases.tokens(cfg, 60, 40 + k)
        first, second = ("a", "b") if k % 2 else ("b", "a")
        n = {"a": 40, "b": 30}
        got = cases.replay(e, {"a": a, "b": b},
                           [[(first, n[first]), (second, n[second])], [("b", 29), ("a", 60)],
                            [("a", 30), ("b", 1)]])
        assert cases.model_error(got["a"], cases.expected("mixed", a), F32) < 1
        assert cases.model_error(got["b"], cases.expected("mixed", b), F32) < 1


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [1, 2, 3, 17])
def test_first_tokens(device, dtype, n):
    """The start of a sequence: convolutions and states begin with nothing."""
    # one token's rounding may choose another expert where choices are close
    name = "mixed" if dtype == F32 else "odd"
    toks = cases.tokens(cases.CONFIGS[name], n, 7)
    want = cases.expected(name, toks)
    for sizes in ([n], [1], [2, 1]):
        e = engine(name, device, dtype)
        got = cases.replay(e, {"r": toks}, [[("r", k)] for k in cases.cut(n, sizes)])
        assert cases.model_error(got["r"], want, dtype) < 1


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(device, dtype):
    toks = cases.tokens(cases.CONFIGS["mixed"], 330, 8)
    want = cases.expected("mixed", toks)
    e = engine("mixed", device, dtype)
    got = cases.replay(e, {"r": toks}, [[("r", 5)]] + [[("r", 1)]] * 325)
    assert cases.model_error(got["r"], want, dtype) < 1


@pytest.mark.parametrize("device", DEVICES)
def test_long_prompt(device):
    """Several spans of the scan and several windows, whole and cut."""
    toks = cases.tokens(cases.CONFIGS["mixed"], 700, 9)
    want = cases.expected("mixed", toks)
    e = engine("mixed", device, F32, max_tokens=768)
    for sizes in ([700], [300, 129, 2, 269], [SPAN]):
        got = cases.replay(e, {"r": toks}, [[("r", n)] for n in cases.cut(700, sizes)])
        assert cases.model_error(got["r"], want, F32) < 1, sizes


@pytest.mark.gpu
def test_kernels_refuse_bad_operands():
    ext = ragged.hip_ragged()
    assert ext is not None
    _, batch = batch_of({"a": (0, 20)}, "cuda")
    dev = dict(device="cuda")
    ints = (batch.cu, batch.pos0, batch.slots)
    h = torch.zeros(20, 64, **dev)
    w, hist, out = torch.zeros(4, 64, **dev), torch.zeros(2, 3, 64, **dev), torch.zeros(20, 64, **dev)
    conv = lambda **k: ext.conv_short(*{**dict(  # noqa: E731
        h=h, w=w, b=None, hist=hist, out=out), **k}.values(), *ints, 1, 20, False, False)
    one = torch.ones((), **dev)
    sh = ScanShape(8, 16, 4)
    s = dict(x=torch.zeros(20, 8, **dev), z=torch.zeros(20, 8, **dev), dt=torch.zeros(20, 8, **dev),
             b=torch.zeros(8, **dev), bc=torch.zeros(20, sh.width, **dev),
             A=torch.zeros(16, 8, **dev), D=torch.zeros(8, **dev),
             state=torch.zeros(2, 1, 16, 8, **dev), out=torch.zeros(20, 8, **dev))
    scan = lambda part=16, **k: ext.scan_short(  # noqa: E731
        *{**s, **k}.values(), *ints, 1, 20, part, 1, *sh.columns[1:])
    idx = torch.zeros(20, 2, dtype=torch.int32, **dev)
    tiles = torch.zeros(4, 3, dtype=torch.int32, **dev)
    up = torch.zeros(3, 64, 64, **dev)
    router = torch.zeros(1, 2, 64, 8, **dev)
    tab = torch.zeros(64, 8, **dev)
    pool = torch.zeros(640, 2 * 48, **dev)
    sizes = (4, 2, 32, 16, 32, 16, batch.tok_pos, batch.tok_entry, batch.pages, 20)
    y = torch.zeros(20, 4 * 32 + 2 * 32 + 2 * 16, **dev)
    turn = lambda cos, sin: ext.grouped_turn(  # noqa: E731
        y, None, None, 1e-6, True, cos, sin, None, None, pool, *sizes, True)
    soft, none = (False, True), (0, 0.0, 0.0)
    conv(), scan(), turn(tab, tab)
    bad = (
        lambda: conv(w=torch.zeros(9, 64, **dev)),
        lambda: conv(hist=hist[:, :2].contiguous()),
        lambda: conv(out=torch.zeros(20, 32, **dev)),
        lambda: conv(w=w.bfloat16()),
        lambda: ext.norm_conv_short(h, None, None, torch.ones(64, **dev), 1e-6, w, hist, out, *ints, 1, 20),
        lambda: ext.norm_conv_short(h, h[:10], None, one, 1e-6, w, hist, out, *ints, 1, 20),
        lambda: scan(part=24),
        lambda: scan(A=torch.zeros(12, 8, **dev)),
        lambda: scan(bc=torch.zeros(20, 32, **dev)),
        lambda: scan(state=torch.zeros(2, 1, 8, 16, **dev)),
        lambda: ext.expert_route(h[:, :32], router, torch.zeros(5, **dev), 5, 4, 2, *soft),
        lambda: ext.expert_route(h, router, torch.zeros(17, **dev), 5, 4, 2, *soft),
        lambda: ext.expert_route(h, router, torch.zeros(17, **dev), 17, 4, 2, *soft),
        lambda: ext.expert_route(h, router, torch.zeros(5, **dev), 5, 4, 6, *soft),
        lambda: ext.expert_plan(idx, idx, torch.zeros(1, 3, dtype=torch.int32, **dev), None, 3, 16),
        lambda: ext.expert_gemm(h, idx.view(-1), tiles, up, None, 32, 40, *none),
        lambda: ext.expert_gemm(h, None, tiles, up, None, 16, 40, *none),
        lambda: ext.expert_gemm(h[:, :32], idx.view(-1), tiles, up, None, 16, 40, *none),
        lambda: ext.token_gate(h, router, torch.zeros(20, 17, **dev)),
        lambda: turn(tab[:, :4], tab[:, :4]),
        lambda: turn(torch.zeros(64, 20, **dev), torch.zeros(64, 20, **dev)),
        lambda: turn(tab, None),
        lambda: ext.grouped_attn_short(
            torch.zeros(20, 4, 32, **dev), None, pool, torch.zeros(20, 64, **dev), batch.cu,
            batch.pos0, batch.pages, 1, 20, 20, 20, 2, 16, 16, 1.0, 0, tab[:, :4].contiguous(),
            tab[:, :4].contiguous(), batch.tok_pos),
    )
    for i, call in enumerate(bad):
        with pytest.raises(RuntimeError):
            call()
            raise AssertionError(i)


@pytest.mark.gpu
def test_bf16_matches_cpu_path_on_kernel_shapes():
    """The shapes a real model has, GPU kernels against the torch path."""
    g = torch.Generator().manual_seed(9)
    for layer in (cases.attention(16, 4, 128, 128, 512), cases.mamba(512, 16, 32, 4)):
        a = Mixer(layer, 256, BF16, "cuda")
        b = Mixer(layer, 256, F32, "cpu", a.w)
        h = torch.randn(1100, 256, generator=g)
        want = b.run(h.bfloat16().float(), [1100])
        for sizes in ([1100], [1000, 1], [300, 128, 16]):
            assert cases.error(a.run(h, sizes), want) < 3e-2
