"""Lepizen against the plain oracle: mechanisms alone, then the batch engine."""

import math

import pytest
import torch

import lepizen_cases as cases
import lepizen_oracle as oracle
from mlx_sharding_amd.ops import ragged
from mlx_sharding_amd.ops.paged import PagedState, RaggedBatch, RowSpec
from mlx_sharding_amd.ops.ragged import GroupedShape
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


# ---------------------------------------------------------------------------
# Mechanisms alone
# ---------------------------------------------------------------------------

def test_oracle_forms_agree():
    """The row form of the oracle's attention is the token form."""
    torch.manual_seed(0)
    q, k, v = torch.randn(9, 6, 5), torch.randn(9, 2, 5), torch.randn(9, 2, 3)
    q, k, v, sink = (t.double() for t in (q, k, v, torch.randn(6)))
    assert torch.allclose(oracle.attend(q, k, v, sink, 0.7),
                          oracle.attend_rows(q, k, v, sink, 0.7))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [40, 97, 1024, 2500, 9000])
@pytest.mark.parametrize("mult", [1.0, 0.35])
def test_residual_update(device, dtype, W, mult):
    """x + mult * y without a norm of y, then the next norm."""
    torch.manual_seed(0)
    eps = 0.05  # large, so that a misplaced eps shows
    x, wn = torch.randn(5, W), (1 + 0.3 * torch.randn(W)).to(dtype)
    wide = (torch.randn(5, W + 8) * 3).to(dtype)
    for y in (wide[:, :W].contiguous(), wide[:, :W]):
        want_x = x.double() + mult * y.double()
        want_h = oracle.rms_norm(want_x, wn.double(), eps)
        xd = x.clone().to(device)
        yd = wide.to(device)[:, :W] if y.stride(0) != W else y.to(device)
        h = ragged.add_norm(xd, yd, None, wn.to(device), eps, 0.0, dtype, mult)
        assert h.dtype == dtype
        assert cases.error(xd, want_x) < 1e-6
        assert cases.error(h, want_h) < (1e-6 if dtype == F32 else 4e-3)
        xd = x.clone().to(device)
        assert ragged.add_norm(xd, yd, None, None, eps, 0.0, dtype, mult) is None
        assert cases.error(xd, want_x) < 1e-6


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("C", [1, 33, 64, 4096])
def test_gelu(device, dtype, C):
    x = torch.cat([torch.linspace(-9, 9, 3 * C), torch.zeros(C)]).view(4, C).to(dtype)
    want = oracle.gelu(x.double())
    got = ragged.gelu(x.to(device)).double().cpu()
    if dtype == F32:
        assert float((got - want).abs().max()) < 1e-6
        if C >= 33:     # the tanh form is another function
            other = torch.nn.functional.gelu(x.double(), approximate="tanh")
            assert float((other - want).abs().max()) > 1e-4
    else:
        assert bool(((got - want).abs() <= 4e-3 * want.abs() + 1e-6).all())
    # into and out of slices of wider rows
    wide = torch.zeros(4, C + 24, dtype=dtype, device=device)
    wide[:, 8: 8 + C] = x.to(device)
    out = torch.full((4, C + 11), 7.0, dtype=dtype, device=device)
    ragged.gelu(wide[:, 8: 8 + C], out[:, 3: 3 + C])
    assert torch.allclose(out[:, 3: 3 + C].double().cpu(), got, rtol=8e-3, atol=1e-6)
    assert bool((out[:, :3] == 7).all()) and bool((out[:, 3 + C:] == 7).all())


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("scale,limit", [(0.5, 3.0), (1.0, 1.0), (2.5, 30.0)])
def test_cap_logits(device, dtype, scale, limit):
    z = (torch.linspace(-40, 40, 3 * 101).view(3, 101)).to(dtype)
    got = ragged.cap_logits(z.to(device), scale, limit)
    assert got.dtype == F32
    want = oracle.cap(z.double(), scale, limit)
    assert float((got.double().cpu() - want).abs().max()) < 2e-6 * limit


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff", [64, 33, 1])
def test_mlp(device, dtype, ff):
    from mlx_sharding_amd.models.mixers import MLP
    torch.manual_seed(0)
    w = {"m.up": (torch.randn(ff, 48) * 48 ** -0.5).to(dtype),
         "m.down": (torch.randn(48, ff) * ff ** -0.5).to(dtype)}
    m = MLP(48, ff, "gelu", dtype)
    m.load_state_dict({k[2:] + ".weight": v for k, v in w.items()})
    h = (torch.randn(7, 48) * 2).to(dtype)
    want = oracle.mlp(h.double(), {k: v.double() for k, v in w.items()}, "m.")
    assert cases.error(m.to(device)(h.to(device)), want) < (2e-6 if dtype == F32 else 2e-2)


def test_page_layout():
    """Every (page, key, head, dimension) has a place of its own, in fragments
    of 64 lanes x 8 elements."""
    sh = GroupedShape(4, 2, 40, 24)
    assert (sh.dimp, sh.vdp, sh.width) == (64, 32, 192)
    rows = torch.arange(2 * 64 * sh.width).view(-1, sh.width)
    k = sh.keys(rows).reshape(2, 64, 2, 64)
    v = sh.values(rows).reshape(2, 64, 2, 32)
    assert torch.cat([k.reshape(-1), v.reshape(-1)]).unique().numel() == rows.numel()
    page, key, g, d = 1, 37, 1, 43
    head = 64 * (64 + 32)
    lane = d // 8 % 4 * 16 + key % 16
    assert int(k[page, key, g, d]) == ((page * 2 + g) * head
                                       + ((key // 16 * 2 + d // 32) * 64 + lane) * 8 + d % 8)
    d = 21
    lane = key // 4 % 4 * 16 + d % 16
    assert int(v[page, key, g, d]) == (
        (page * 2 + g) * head + 64 * 64
        + ((d // 16 * 2 + key // 32) * 64 + lane) * 8 + key // 16 % 2 * 4 + key % 4)


def batch_of(portions, device, max_tokens=640):
    """A state with one poisoned layer, its requests {id: (held, new)}."""
    lens = {r: p + n for r, (p, n) in portions.items()}
    state = PagedState([], max_tokens, 8, F32, device)
    for r, n in lens.items():
        state.admit(r)
        state.reserve(r, n)
        state.live[r].length = portions[r][0]
    return state, RaggedBatch([(state.live[r], n) for r, (_, n) in portions.items()], device)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,V", [(6, 2, 24, 40), (2, 1, 17, 5), (4, 4, 128, 64),
                                     (3, 3, 272, 8), (40, 5, 72, 16),
                                     (24, 4, 256, 8), (64, 8, 160, 24)])
def test_append(device, dtype, H, G, D, V):
    """Queries and keys normed over their whole rows, values blended, each in
    its slot; slots before a portion's start keep what they hold."""
    portions = {"a": (60, 1), "b": (3, 70), "c": (0, 16), "d": (130, 17), "e": (64, 64)}
    state, batch = batch_of(portions, device)
    sh = GroupedShape(H, G, D, V)
    torch.manual_seed(0)
    from mlx_sharding_amd.ops.paged import LayerStore
    store = LayerStore(RowSpec(sh.width), state.n_pages, 1, dtype, device)
    store.rows.fill_(float("nan"))
    N = batch.n_tokens
    y = (torch.randn(N, (H + G) * D + G * V + 3) * 2).to(dtype)
    y = torch.nn.functional.pad(y, (0, -y.shape[1] % 8))
    wq, wk = (1 + 0.3 * torch.randn(H * D)).to(dtype), (1 + 0.3 * torch.randn(G * D)).to(dtype)
    vmix, first = torch.tensor(0.3).to(dtype), torch.randn(N, G * V).to(dtype)
    eps = 0.3
    q64, k64, v64 = y.double()[:, : (H + G) * D + G * V].split([H * D, G * D, G * V], 1)
    qn, kn = oracle.rms_norm(q64, wq.double(), eps), oracle.rms_norm(k64, wk.double(), eps)
    vm = oracle.mixed_values(v64, first.double(), vmix.double())
    tol = 1e-6 if dtype == F32 else 8e-3
    on = lambda t: None if t is None else t.to(device)  # noqa: E731
    for want_q, want_k, want_v, args in (
            (qn, kn, vm, (wq, wk, eps, vmix, first)),
            (q64, k64, v64, (None, None, eps, None, None))):
        wq_, wk_, eps_, vmix_, first_ = args
        q = ragged.grouped_append(y.to(device), on(wq_), on(wk_), eps_, on(vmix_),
                                  on(first_), store, sh, batch)
        assert q.shape == (N, H, sh.dimp) and bool((q[..., D:] == 0).all())
        assert cases.error(q[..., :D].reshape(N, -1), want_q) < tol
        for t0, n, p0, held in batch.host:
            pages = torch.tensor(held.pages, device=device)
            k = sh.keys(store.rows)[pages].reshape(-1, G, sh.dimp)
            v = sh.values(store.rows)[pages].reshape(-1, G, sh.vdp)
            kk, vv = k[p0: p0 + n], v[p0: p0 + n]
            assert bool((kk[..., D:] == 0).all()) and bool((vv[..., V:] == 0).all())
            assert cases.error(kk[..., :D].reshape(n, -1), want_k[t0: t0 + n]) < tol
            assert cases.error(vv[..., :V].reshape(n, -1), want_v[t0: t0 + n]) < tol
            assert bool(torch.isnan(k[:p0]).all()) and bool(torch.isnan(v[:p0]).all())


class Mixer:
    """The attention of one layer with its storage: feed portions, compare."""

    def __init__(self, layer, width, dtype, device, w=None, seed=0, eps=1e-5):
        cfg = cases.config(width, 8, [layer], eps)
        self.w = w or cases.weights(cfg, seed)
        self.model = cases.build(cfg, self.w, device, dtype)
        self.mix = self.model.l0.mix
        self.layer, self.dtype, self.device, self.eps = layer, dtype, device, eps

    def want(self, h, first=None, w=None):
        w = {k: v.double() for k, v in (w or self.w).items()}
        if first is not None:
            first = first.to(self.dtype).double()
        return oracle.attention(h.to(self.dtype).double(), w, "l0.mix.",
                                self.layer["mixer"], self.eps, first)[0]

    def run(self, h, sizes, first=None):
        """h [T, width] in portions of these sizes (the last one repeated)."""
        T = h.shape[0]
        state = self.model.make_state(T + 64, 2)
        cases.poison(state)
        state.admit("other")       # so that the pages are not the first
        state.reserve("other", 1)
        held = state.admit("x")
        outs, at = [], 0
        for n in cases.cut(T, sizes):
            state.reserve("x", at + n)
            batch = RaggedBatch([(held, n)], self.device)
            part = lambda t: t[at: at + n].to(self.device, self.dtype)  # noqa: E731
            y, raw = self.mix(part(h), batch, state.layers[0],
                              None if first is None else part(first))
            assert raw.shape == (n, self.mix.v.out_features)
            outs.append(y.cpu())
            at += n
            held.length = at
        return torch.cat(outs)


LAYERS = {
    "grouped": cases.layer(6, 2, 24, 40),
    "one": cases.layer(1, 1, 8, 8),
    "own keys": cases.layer(5, 5, 32, 16),
    "shared keys": cases.layer(20, 1, 16, 24),
    "odd": cases.layer(6, 3, 17, 5, scale=0.5),
    "64/128": cases.layer(4, 2, 64, 128),
    "128/64": cases.layer(4, 2, 128, 64),
    "128": cases.layer(8, 2, 128, 128),
    "96/256": cases.layer(2, 2, 96, 256),
    "256/80": cases.layer(4, 2, 256, 80),
    "192": cases.layer(4, 1, 192, 192),
    "too wide for prompts": cases.layer(4, 2, 272, 272),
    "widest": cases.layer(2, 1, 512, 512),
    "wide keys": cases.layer(2, 1, 300, 48),
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", LAYERS)
def test_attention(device, dtype, kind):
    m = Mixer(LAYERS[kind], 64, dtype, device, eps=0.2)
    g = torch.Generator().manual_seed(3)
    h = torch.randn(150, 64, generator=g)
    first = torch.randn(150, m.mix.v.out_features, generator=g)
    tol = 1e-5 if dtype == F32 else 2e-2
    for f in (None, first):
        want = m.want(h, f)
        for sizes in ([150], [1], [64, 17, 2, 60], [16], [2, 3, 129]):
            assert cases.error(m.run(h, sizes, f), want) < tol, sizes


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_sink(device, dtype):
    """Sinks far above, among and far below the scores; each head its own,
    counted once however the keys are split, and not scaled."""
    layer = cases.layer(6, 2, 32, 32, scale=0.05)
    w = cases.weights(cases.config(64, 8, [layer]))
    w["l0.mix.sink"] = torch.tensor([9.0, 5.5, 0.0, -40.0, 3.0, 7.0]).bfloat16()
    m = Mixer(layer, 64, dtype, device, w)
    h = torch.randn(600, 64, generator=torch.Generator().manual_seed(3))
    want = m.want(h)
    for change in (lambda s: s - 40, lambda s: s * 0.05, lambda s: s + math.log(2),
                   lambda s: s.flip(0)):
        other = dict(w)
        other["l0.mix.sink"] = change(w["l0.mix.sink"].float()).bfloat16()
        assert cases.error(m.want(h, w=other), want) > 0.1
    tol = 1e-5 if dtype == F32 else 2e-2
    for sizes in ([600], [590, 1], [64, 17, 2, 300], [16]):
        assert cases.error(m.run(h, sizes), want) < tol, sizes


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_norms_span_all_heads(device, dtype):
    """One head loud, the others quiet: a norm per head would level them."""
    layer = cases.layer(4, 2, 32, 16, scale=0.1)
    w = cases.weights(cases.config(64, 8, [layer]))
    for n, rows in (("q", 32), ("k", 32)):
        t = w[f"l0.mix.{n}"].clone()
        t[rows:] *= 0.15
        w[f"l0.mix.{n}"] = t
    w["l0.mix.sink"] = torch.zeros(4).bfloat16()
    m = Mixer(layer, 64, dtype, device, w)
    h = torch.randn(90, 64, generator=torch.Generator().manual_seed(3))
    want = m.want(h)
    w64 = {k: v.double() for k, v in w.items()}
    x = h.to(dtype).double()

    def each(t, weight, n):
        t = t.view(90, n, 32)
        t = t / torch.sqrt(t.pow(2).mean(-1, keepdim=True) + m.eps)
        return t * weight.view(n, 32)
    per_head = oracle.attend_rows(
        each(x @ w64["l0.mix.q"].T, w64["l0.mix.q.norm"], 4),
        each(x @ w64["l0.mix.k"].T, w64["l0.mix.k.norm"], 2),
        (x @ w64["l0.mix.v"].T).view(90, 2, 16), w64["l0.mix.sink"], 0.1)
    assert cases.error(per_head.reshape(90, -1) @ w64["l0.mix.o"].T, want) > 0.1
    for sizes in ([90], [1]):
        assert cases.error(m.run(h, sizes), want) < (1e-5 if dtype == F32 else 2e-2)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_single_key_stands_out(device, dtype):
    """Queries of one head that look for one key: the first token, keys far
    back, at page and tile borders and next to them, the token itself.  The key
    carries most of the weight, so a missing or misplaced one cannot hide."""
    layer = cases.layer(4, 2, 32, 24, scale=0.3)
    mx, D = layer["mixer"], 32
    m = Mixer(layer, 160, dtype, device)
    w = {k: v.double() for k, v in m.w.items()}
    T, head = 700, 2
    h = torch.randn(T, 160, generator=torch.Generator().manual_seed(5), dtype=torch.float64)
    asks = {40: 31, 41: 32, 66: 63, 67: 64, 100: 0, 140: 126, 129: 127, 130: 128,
            191: 127, 192: 15, 193: 16, 259: 31, 258: 47, 300: 1, 319: 255,
            320: 256, 449: 0, 500: 3, 513: 383, 514: 384, 640: 63, 641: 64,
            690: 511, 698: 512, 699: 0}
    keys = oracle.rms_norm(h @ w["l0.mix.k"].T, w["l0.mix.k.norm"], m.eps).view(T, 2, D)[:, head // 2]
    wq = w["l0.mix.q"] * 1.0
    for q, k in asks.items():
        want = torch.zeros(4 * D, dtype=torch.float64)
        want[head * D: (head + 1) * D] = keys[k] / w["l0.mix.q.norm"][head * D: (head + 1) * D]
        h[q] = torch.linalg.lstsq(wq, want[:, None]).solution[:, 0] * 10
    h = h.to(dtype).double()
    x = oracle.rms_norm(h @ w["l0.mix.q"].T, w["l0.mix.q.norm"], m.eps).view(T, 4, D)[:, head]
    keys = oracle.rms_norm(h @ w["l0.mix.k"].T, w["l0.mix.k.norm"], m.eps).view(T, 2, D)[:, head // 2]
    for q, k in asks.items():
        s = keys[: q + 1] @ x[q] * mx["scale"]
        assert torch.softmax(s, 0)[k] > 0.5, (q, k)
    want = m.want(h)
    tol = 2e-5 if dtype == F32 else 3e-2
    rows = sorted(asks)
    for sizes in ([T], [90, 1], [T - 40, 1], [128, 128, 2], [97, 3], [16], [63, 2, 65]):
        got = m.run(h, sizes)
        assert cases.error(got[rows], want[rows]) < tol, sizes


@pytest.mark.parametrize("device", DEVICES)
def test_future_is_not_seen(device):
    """A loud token at i + 1 does not change what token i gives."""
    m = Mixer(cases.layer(4, 2, 32, 16), 64, F32, device)
    h = torch.randn(140, 64, generator=torch.Generator().manual_seed(3))
    base = m.run(h, [140])
    for i in (0, 15, 16, 31, 62, 63, 64, 127, 128):
        loud = h.clone()
        loud[i + 1:] = 50 * torch.randn(139 - i, 64)
        assert torch.equal(m.run(loud, [140])[: i + 1], base[: i + 1]), i


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff", [None, 30, 64])
def test_parallel_block(device, dtype, ff):
    """Both sublayers read the same rows; their sum comes back."""
    layer = cases.layer(3, 3, 20, 10, ff=ff)
    m = Mixer(layer, 48, dtype, device)
    h = torch.randn(30, 48, generator=torch.Generator().manual_seed(3))
    want = m.want(h)
    if ff is not None:
        want = want + oracle.mlp(h.to(dtype).double(),
                                 {k: v.double() for k, v in m.w.items()}, "l0.mlp.")
    state = m.model.make_state(64, 1)
    held = state.admit(0)
    state.reserve(0, 30)
    batch = RaggedBatch([(held, 30)], device)
    got, raw = m.model.l0(h.to(device, dtype), batch, state.layers[0], None)
    assert cases.error(got, want) < (1e-5 if dtype == F32 else 2e-2)
    v = h.to(dtype).double() @ m.w["l0.mix.v"].double().T
    assert cases.error(raw, v) < (1e-5 if dtype == F32 else 1e-2)


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
    cfg, w = cases.CONFIGS["mixed"], cases.weights(cases.CONFIGS["mixed"])
    toks = cases.tokens(cfg, 60)
    want = cases.expected("mixed", toks)

    def off(change, **constants):
        other = {k: v.clone() for k, v in w.items()}
        change(other)
        return cases.error(oracle.forward({**cfg, **constants}, other, toks), want)

    none = lambda t: None  # noqa: E731
    assert off(none) == 0
    for i in range(5):
        assert off(lambda t: t[f"l{i}.mix.sink"].fill_(-50.0)) > 0.04, i
    for i in (3, 4):
        assert off(lambda t: t[f"l{i}.mix.vmix"].fill_(0.0)) > 0.04, i
    # the first mixing layer has nothing to mix in
    assert off(lambda t: t["l1.mix.vmix"].fill_(0.0)) == 0
    for constants in (dict(residual_mult=0.5), dict(logit_scale=0.6),
                      dict(logit_softcap=7.0), dict(norm={"eps": 0.1})):
        assert off(none, **constants) > 0.01, constants


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
def test_layers(device, dtype):
    """The residual stream after every layer."""
    cfg = cases.CONFIGS["mixed"]
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
@pytest.mark.parametrize("name", ["mixed", "wide"])
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
    pages in another order each time."""
    e = engine("mixed", device, F32, max_tokens=256, max_requests=2)
    cfg = cases.CONFIGS["mixed"]
    for k in range(4):
        a, b = cases.tokens(cfg, 130, 20 + k), cases.tokens(cfg, 60, 40 + k)
        got = cases.replay(e, {"a": a, "b": b},
                           [[("a", 40), ("b", 30)], [("b", 29), ("a", 60)],
                            [("a", 30), ("b", 1)]])
        assert cases.model_error(got["a"], cases.expected("mixed", a), F32) < 1
        assert cases.model_error(got["b"], cases.expected("mixed", b), F32) < 1


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [1, 2, 3, 17])
def test_first_tokens(device, dtype, n):
    """The start of a sequence, where the sink has the most weight."""
    toks = cases.tokens(cases.CONFIGS["mixed"], n, 7)
    want = cases.expected("mixed", toks)
    for sizes in ([n], [1], [2, 1]):
        e = engine("mixed", device, dtype)
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


@pytest.mark.gpu
def test_kernels_refuse_bad_operands():
    ext = ragged.hip_ragged()
    assert ext is not None
    state, batch = batch_of({"a": (0, 20)}, "cuda")
    sh = GroupedShape(4, 2, 32, 16)
    y = torch.zeros(20, 4 * 32 + 2 * 32 + 2 * 16, device="cuda")
    w = torch.ones(128, device="cuda")
    pool = torch.zeros(512, sh.width, device="cuda")
    sizes = (4, 2, 32, 16, 32, 16)
    where = (batch.tok_pos, batch.tok_entry, batch.pages)
    bad = (
        lambda: ext.grouped_append(y[:, :64], w, None, 1e-6, None, None, pool, *sizes, *where, 0),
        lambda: ext.grouped_append(y, w[:64], None, 1e-6, None, None, pool, *sizes, *where, 0),
        lambda: ext.grouped_append(y, w, None, 1e-6, None, y[:, :32], pool, *sizes, *where, 0),
        lambda: ext.grouped_append(y, w, None, 1e-6, None, None, pool[:, 1:], *sizes, *where, 0),
        lambda: ext.grouped_append(y, w.bfloat16(), None, 1e-6, None, None, pool, *sizes, *where, 0),
        lambda: ext.grouped_append(y, w, None, 1e-6, None, None, pool, *sizes, *where, 21),
        lambda: ext.grouped_attn_long(
            torch.zeros(20, 4, 288, device="cuda"), None, torch.zeros(512, 2 * 304, device="cuda"),
            torch.zeros(20, 64, device="cuda"), batch.tiles, batch.cu, batch.pos0, batch.pages,
            2, 16, 16, 1.0),
        lambda: ext.gelu(y, y[:10]),
        lambda: ext.cap_logits(y, 1.0, 0.0),
    )
    for call in bad:
        with pytest.raises(RuntimeError):
            call()
    with pytest.raises(ValueError):
        GroupedShape(6, 4, 32, 32)


@pytest.mark.gpu
def test_bf16_matches_cpu_path_on_kernel_shapes():
    """The shapes a real model has, GPU kernels against the torch path."""
    layer = cases.layer(16, 4, 128, 128)
    g = Mixer(layer, 256, BF16, "cuda")
    c = Mixer(layer, 256, F32, "cpu", g.w)
    h = torch.randn(1500, 256, generator=torch.Generator().manual_seed(9))
    want = c.run(h.bfloat16().float(), [1500])
    for sizes in ([1500], [1400, 1], [300, 128, 16]):
        assert cases.error(g.run(h, sizes), want) < 2e-2
