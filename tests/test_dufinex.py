"""Dufinex against the plain oracle: mechanisms alone, then the batch engine."""

import copy
import math

import pytest
import torch
import torch.nn.functional as F

import dufinex_cases as cases
import dufinex_oracle as oracle
from mlx_sharding_amd.models.mixers import (BiasedMLP, GatedDelta,
                                            GroupedAttention, RoutedExperts)
from mlx_sharding_amd.ops import experts, ragged
from mlx_sharding_amd.ops.experts import ExpertShape, Routing
from mlx_sharding_amd.ops.paged import (CHUNK, LayerStore, PagedState,
                                        RaggedBatch, RowSpec, StateSpec)
from mlx_sharding_amd.ops.ragged import (ClampedGLU, DeltaShape, GroupedShape,
                                         Rotary, Turns)
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
    g = torch.Generator().manual_seed(0)
    q, k, v = (torch.randn(11, n, 5, generator=g).double() for n in (6, 2, 2))
    sink = torch.tensor([-3.0, 0.0, 0.5, 1.0, 2.0, 9.0]).double()
    assert torch.allclose(oracle.attend(q, k, v, 0.7, sink),
                          oracle.attend_rows(q, k, v, 0.7, sink))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("C", [64, 33, 1, 520])
@pytest.mark.parametrize("limit", [0.5, 1.0, 7.0])
def test_clamped_glu(device, dtype, C, limit):
    """Both sides of both limits, in columns of wider rows."""
    g = torch.Generator().manual_seed(1)
    rows = (torch.randn(9, 2 * C + 8, generator=g) * 6).to(dtype)
    rows[0, :2] = torch.tensor([-60.0, 60.0])
    on = rows.to(device)
    got = ClampedGLU(limit)(on[:, :C], on[:, C: 2 * C])
    assert got.dtype == dtype and got.shape == (9, C)
    gate, up = rows[:, :C].double(), rows[:, C: 2 * C].double()
    want = oracle.clamped_glu(gate, up, limit)
    tol = 1e-6 if dtype == F32 else 8e-3
    assert bool(((got.double().cpu() - want).abs() <= tol * (1 + want.abs())).all())
    if C > 60 and limit <= 1:      # the gate has no lower limit, and one is added to up
        low = torch.clamp(gate, -limit, limit)
        assert cases.error(oracle.clamped_glu(low, up, limit), want) > 0.02
        assert cases.error(low * oracle.sigmoid(1.702 * low) * up, want) > 0.1


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff", [64, 33, 1])
def test_mlp_with_biases(device, dtype, ff):
    g = torch.Generator().manual_seed(2)
    m = BiasedMLP(48, ff, ClampedGLU(1.5), dtype)
    for p in m.parameters():
        p.data = (torch.randn(p.shape, generator=g) * 0.2).to(dtype)
    w = {}
    for n in ("gate", "up", "down"):
        w[f"m.{n}"], w[f"m.{n}.b"] = (t.double() for t in (
            getattr(m, n).weight, getattr(m, n).bias))
    h = (torch.randn(7, 48, generator=g) * 2).to(dtype)
    m.to(device).prepare()
    # rows of the residual's copy are wider than the model
    wide = F.pad(h, (0, 16)).to(device)[:, :48]
    want = oracle.dense(h.double(), w, "m.", 1.5)
    tol = 2e-6 if dtype == F32 else 2e-2
    assert cases.error(m(wide), want) < tol
    # the last bias goes with the residual update
    x = torch.randn(7, 48, generator=g)
    y, bias = m.rows(wide)
    xd = x.clone().to(device)
    ragged.add_norm(xd, y, None, None, 1e-5, 0.0, dtype, y_bias=bias)
    assert cases.error(xd, x.double() + want) < tol
    xd = x.clone().to(device)
    ragged.add_norm(xd, y, bias, None, 1e-2, 0.0, dtype, y_bias=bias)
    assert cases.error(xd, x.double() + oracle.rms(want, 1e-2) * w["m.down.b"]) < tol


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [40, 97, 1024, 2500, 9000])
@pytest.mark.parametrize("top", [0, 1, 5])
def test_norm_of_the_output(device, dtype, W, top):
    """What is added is normed; the copy that follows is the residual itself,
    padded; with ``where``, rows are summed first."""
    g = torch.Generator().manual_seed(3)
    n, eps = 6, 0.05     # large, so that a misplaced eps shows
    x = torch.randn(n, W, generator=g)
    rows = (torch.randn(n * max(top, 1), F.pad(x, (0, -W % 8)).shape[1], generator=g) * 3).to(dtype)
    w = (1 + 0.3 * torch.randn(W, generator=g)).to(dtype)
    where, y = None, rows[:, :W].double()
    if top:
        where = torch.randperm(n * top, generator=g).view(n, top).int()
        y = y[where.long()].sum(1)
    want = x.double() + oracle.rms(y, eps) * w.double()
    on = lambda t: None if t is None else t.to(device)  # noqa: E731
    yd = on(rows) if top else on(rows)[:, :W]
    xd = on(x.clone())
    copied = ragged.add_norm(xd, yd, on(w), None, eps, 0.0, dtype, where=on(where), copy=True,
                             pad_to=64)
    assert copied.dtype == dtype and copied.shape == (n, -(-W // 64) * 64)
    assert cases.error(xd, want) < 1e-6
    assert torch.equal(copied[:, :W], xd.to(dtype)) and bool((copied[:, W:] == 0).all())
    xd = on(x.clone())
    h = ragged.add_norm(xd, yd, on(w), on(w), eps, 0.0, dtype, where=on(where), copy=True)
    assert cases.error(xd, want) < 1e-6
    assert cases.error(h, oracle.rms(want, eps) * w.double()) < (1e-6 if dtype == F32 else 4e-3)
    # no sublayer: the residual stays, only the copy is made
    before = xd.clone()
    copied = ragged.add_norm(xd, None, None, None, eps, 0.0, dtype, copy=True, pad_to=8)
    assert torch.equal(xd, before) and torch.equal(copied[:, :W], xd.to(dtype))
    copied.fill_(0)
    assert torch.equal(xd, before)      # a copy also in 32-bit


SHAPES = {
    "usual": ExpertShape(96, 80, 12, 0, 4),
    "one each": ExpertShape(64, 64, 16, 0, 1),
    "odd": ExpertShape(51, 33, 5, 0, 3),
    "all": ExpertShape(40, 8, 3, 0, 3),
    "one": ExpertShape(17, 1, 1, 0, 1),
    "many": ExpertShape(128, 24, 190, 0, 9),
    "wide": ExpertShape(72, 330, 4, 0, 2),
}


def routed(sh, dtype, seed, limit=1.0):
    g = torch.Generator().manual_seed(seed)
    m = RoutedExperts(sh.width, sh.ff, sh.experts, 0, sh.top, dtype, glu=ClampedGLU(limit),
                      routing=Routing("sigmoid", False, True), correction=False)
    for t, gain in ((m.gate.weight, 2 * sh.width ** -0.5), (m.up.weight, 2 * sh.width ** -0.5),
                    (m.down.weight, sh.ff ** -0.5), (m.router.weight, sh.width ** -0.5)):
        t.data = (torch.randn(t.shape, generator=g) * gain).to(dtype)
    return m


def routed_oracle(m, h):
    w = {"m.router": m.router.weight.double()}
    for e in range(m.shape.experts):
        for n in ("gate", "up", "down"):
            w[f"m.e{e}.{n}"] = getattr(m, n).weight[e].double()
    return oracle.experts(h.double(), w, "m.", cases.moe(
        m.shape.ff, m.shape.experts, m.shape.top, m.glu.limit))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", SHAPES)
@pytest.mark.parametrize("n", [1, 15, 70, 400])
def test_experts(device, dtype, kind, n):
    """Few and many tokens per expert: rows to be summed, and the form that
    adds them to a residual."""
    sh = SHAPES[kind]
    m = routed(sh, dtype, n)
    h = torch.randn(n, sh.width, generator=torch.Generator().manual_seed(n)).to(dtype)
    want = routed_oracle(m, h)
    m.to(device)
    hp = F.pad(h, (0, sh.widthp - sh.width)).to(device)
    rows, where = m.rows(hp)
    assert where.shape == (n, sh.top)
    assert sorted(where.flatten().tolist()) == list(range(n * sh.top))
    got = rows.double().cpu()[where.long().cpu()].sum(1)[:, : sh.width]
    tol = 5e-6 if dtype == F32 else 2e-2
    assert cases.error(got, want) < tol
    x = torch.zeros(n, sh.width, device=device)
    m(x, hp)
    assert cases.error(x, want) < tol
    # the parameters still are the experts' own matrices
    assert cases.error(routed_oracle(m.cpu(), h), want) == 0


@pytest.mark.gpu
@pytest.mark.parametrize("tile", [16, 128])
def test_tile_sizes_agree(tile, monkeypatch):
    """Both grouped products on the same few and many tokens."""
    monkeypatch.setattr(ExpertShape, "tile", lambda self, tokens: tile)
    for kind in ("usual", "odd", "many", "wide"):
        for n in (3, 130):
            for dtype in DTYPES:
                test_experts("cuda", dtype, kind, n)


def test_weight_on_the_input_is_not_on_the_output():
    """The gated unit is no linear function, so the place of the weight shows."""
    sh = SHAPES["usual"]
    m = routed(sh, F32, 0)
    h = torch.randn(20, sh.width, generator=torch.Generator().manual_seed(0))
    want = routed_oracle(m, h)
    _, weight = oracle.route(h.double() @ m.router.weight.double().T, sh.top)
    x = torch.zeros(20, sh.width)
    m.routing = Routing("sigmoid", False, False)
    m(x, F.pad(h, (0, sh.widthp - sh.width)))
    assert cases.error(x, want) > 0.1
    m.routing = Routing("sigmoid", True, True)
    x.zero_()
    m(x, F.pad(h, (0, sh.widthp - sh.width)))
    assert cases.error(x, want) > 0.1


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("score,normalize", [("softmax", True), ("softmax", False),
                                             ("sigmoid", True), ("sigmoid", False)])
@pytest.mark.parametrize("corrected", [False, True])
def test_routing(device, dtype, score, normalize, corrected):
    """Scores, weights and the choice.  Logits that all round to a score of 1
    still are in order."""
    W, E, top = 64, 30, 4
    g = torch.Generator().manual_seed(4)
    router = torch.randn(E, W, generator=g).to(dtype)
    h = torch.randn(50, W, generator=g).to(dtype)
    if score == "sigmoid":
        h[:10] *= 8
    corr = torch.randn(E, generator=g).to(dtype) if corrected else None
    z = h.double() @ router.double().T
    s = torch.softmax(z, -1) if score == "softmax" else oracle.sigmoid(z)
    by = s + corr.double() if corrected else z
    idx = torch.topk(by, top, -1).indices
    w = s.gather(-1, idx)
    if normalize:
        w = w / w.sum(-1, keepdim=True)
    sh = ExpertShape(W, 8, E, 0, top)
    routing = Routing(score, normalize)
    packed = experts.pack(router, 64).to(device)
    cd = None if corr is None else corr.to(device)
    if device == "cpu":
        got_i, got_w = experts.route(h, packed, cd, sh, routing)
    else:
        got_i, got_w, _, _ = ragged.hip_ragged().expert_route(
            h.to(device), packed, cd, E, E, top, score == "sigmoid", normalize)
    assert torch.equal(got_i.cpu().long(), idx)
    assert float((got_w.cpu().double() - w).abs().max()) < 1e-5


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
@pytest.mark.parametrize("H,G,D,V", [(6, 2, 24, 40), (2, 1, 18, 6), (4, 4, 128, 64),
                                     (3, 3, 272, 8), (8, 2, 64, 32), (1, 1, 2, 2), (5, 1, 7, 3)])
def test_append(device, dtype, H, G, D, V):
    """Norms per head with weights (and a rotation behind them); each key and
    value in its slot; a layer without keys of its own writes nothing."""
    portions = {"a": (60, 1), "b": (3, 70), "c": (0, 16), "d": (130, 17), "e": (64, 64)}
    state, batch = batch_of(portions, device)
    sh = GroupedShape(H, G, D, V)
    g = torch.Generator().manual_seed(5)
    store = LayerStore(RowSpec(sh.width), state.n_pages, 1, dtype, device)
    N, eps = batch.n_tokens, 0.3
    y = (torch.randn(N, (H + G) * D + G * V + 3, generator=g) * 2).to(dtype)
    y = F.pad(y, (0, -y.shape[1] % 8))
    q, k, v = (t.reshape(N, n, -1) for t, n in zip(
        y.double()[:, : (H + G) * D + G * V].split([H * D, G * D, G * V], 1), (H, G, G)))
    wq, wk = ((1 + 0.4 * torch.randn(D, generator=g)).to(dtype) for _ in "qk")
    want_q, want_k = (oracle.rms(t, eps) * w.double() for t, w in ((q, wq), (k, wk)))
    tol = 2e-6 if dtype == F32 else 8e-3
    on = lambda t: t.to(device)  # noqa: E731
    turns = [None]
    if D % 2 == 0:
        turns.append(Turns(Rotary(2, 100.0).tables(1024, device)))
    for t in turns:
        a, b = want_q, want_k
        if t is not None:
            ang = batch.tok_pos.cpu().double()[:, None]
            c, s = torch.cos(ang), torch.sin(ang)
            rot = lambda x: torch.cat([  # noqa: E731
                (x[..., 0] * c - x[..., 1] * s)[..., None],
                (x[..., 1] * c + x[..., 0] * s)[..., None], x[..., 2:]], -1)
            a, b = rot(a), rot(b)
        store.rows.fill_(float("nan"))
        got = ragged.grouped_append(on(y), on(wq), on(wk), eps, None, None, store, sh, batch, t,
                                    True)
        assert got.shape == (N, H, sh.dimp) and bool((got[..., D:] == 0).all())
        assert cases.error(got[..., :D].reshape(N, -1), a.reshape(N, -1)) < tol
        for t0, n, p0, held in batch.host:
            pages = torch.tensor(held.pages, device=device)
            kk = sh.keys(store.rows)[pages].reshape(-1, G, sh.dimp)
            vv = sh.values(store.rows)[pages].reshape(-1, G, sh.vdp)
            assert bool(torch.isnan(kk[:p0]).all()) and bool(torch.isnan(vv[:p0]).all())
            kk, vv = kk[p0: p0 + n], vv[p0: p0 + n]
            assert bool((kk[..., D:] == 0).all()) and bool((vv[..., V:] == 0).all())
            at = slice(t0, t0 + n)
            assert cases.error(kk[..., :D].reshape(n, -1), b[at].reshape(n, -1)) < tol
            assert cases.error(vv[..., :V].reshape(n, -1), v[at].reshape(n, -1)) < tol
    kept = store.rows.clone()
    got = ragged.grouped_append(on(y)[:, : H * D], on(wq), None, eps, None, None, store, sh,
                                batch, None, True, own=False)
    assert cases.error(got[..., :D].reshape(N, -1), want_q.reshape(N, -1)) < tol
    assert torch.equal(kept.nan_to_num(7.0), store.rows.nan_to_num(7.0))


class Mixer:
    """The mixers of one or more layers with their storage: feed portions,
    compare the last one's output."""

    def __init__(self, layers, width, dtype, device, w=None, seed=0, eps=1e-5):
        layers = layers if isinstance(layers, list) else [layers]
        cfg = cases.config(width, 8, layers, eps)
        self.w = w or cases.weights(cfg, seed)
        self.model = cases.build(cfg, self.w, device, dtype)
        self.layers, self.dtype, self.device, self.eps = layers, dtype, device, eps

    def want(self, h, w=None):
        w = {k: v.double() for k, v in (w or self.w).items()}
        h, i = h.to(self.dtype).double(), len(self.layers) - 1
        mx, pre = self.layers[i]["mixer"], f"l{i}.mix."
        if self.layers[i]["type"] == "channel_delta":
            return oracle.channel_delta(h, w, pre, mx, self.eps)
        src = mx.get("kv_from", i)
        k, v = oracle.keys_values(h, w, f"l{src}.mix.", mx, self.eps)
        return oracle.attention(h, w, pre, mx, self.eps, k, v)

    def run(self, h, sizes):
        """h [T, width] in portions of these sizes (the last one repeated); all
        layers read h."""
        T = h.shape[0]
        state = self.model.make_state(T + 64, 2)
        cases.poison(state)
        state.admit("other")       # so that pages and slot are not the first
        state.reserve("other", 1)
        held = state.admit("x")
        outs, at = [], 0
        for n in cases.cut(T, sizes):
            state.reserve("x", at + n)
            batch = RaggedBatch([(held, n)], self.device)
            x = h[at: at + n].to(self.device, self.dtype)
            for i, layer in self.model.layer_items():
                y = layer.mix(x, batch, state.layers[self.model.row_source(
                    self.model.config, i)])
                y = y if layer.mix.__class__ is GatedDelta else y[0]
            outs.append(y.cpu())
            at += n
            held.length = at
        return torch.cat(outs)


ATTENTIONS = {
    "grouped": cases.attention(6, 2, 24, 40),
    "one": cases.attention(1, 1, 2, 2),
    "own keys": cases.attention(5, 5, 32, 16),
    "shared keys": cases.attention(20, 1, 16, 24),
    "odd": cases.attention(6, 3, 17, 5, 0.9),
    "64/128": cases.attention(4, 2, 64, 128),
    "256/80": cases.attention(4, 2, 256, 80),
    "too wide for prompts": cases.attention(4, 2, 272, 272),
    "widest": cases.attention(2, 1, 512, 512),
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ATTENTIONS)
def test_attention(device, dtype, kind):
    """Head norms, sinks and gates; then a layer on the first one's keys."""
    layer = ATTENTIONS[kind]
    reader = copy.deepcopy(layer)
    reader["mixer"].update(kv_from=0, scale=layer["mixer"]["scale"] * 0.7)
    h = torch.randn(150, 64, generator=torch.Generator().manual_seed(3))
    tol = 1e-5 if dtype == F32 else 4e-2
    for layers in ([layer], [layer, reader]):
        m = Mixer(layers, 64, dtype, device, eps=0.2)
        want = m.want(h)
        for sizes in ([150], [1], [64, 17, 2, 60], [16], [2, 3, 129]):
            assert cases.error(m.run(h, sizes), want) < tol, sizes


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_sink_and_gate(device, dtype):
    """Sinks far above, among and far below the scores, gates open and almost
    shut; each head its own, counted once however the keys are split."""
    layer = cases.attention(6, 2, 32, 32, 0.05)
    w = cases.weights(cases.config(64, 8, [layer]))
    w["l0.mix.sink"] = torch.tensor([9.0, 5.5, 0.0, -40.0, 3.0, 7.0]).bfloat16()
    w["l0.mix.g"] = w["l0.mix.g"] * 4
    m = Mixer(layer, 64, dtype, device, w)
    h = torch.randn(600, 64, generator=torch.Generator().manual_seed(3))
    want = m.want(h)
    for key, change in (("sink", lambda s: s - 40), ("sink", lambda s: s * 0.05),
                        ("sink", lambda s: s + math.log(2)), ("sink", lambda s: s.flip(0)),
                        ("g", lambda s: s * 0), ("g", lambda s: s.flip(0))):
        other = dict(w)
        other["l0.mix." + key] = change(w["l0.mix." + key].float()).bfloat16()
        assert cases.error(m.want(h, other), want) > 0.1
    tol = 1e-5 if dtype == F32 else 5e-2
    for sizes in ([600], [590, 1], [64, 17, 2, 300], [16]):
        assert cases.error(m.run(h, sizes), want) < tol, sizes


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shared", [False, True])
def test_single_key_stands_out(device, dtype, shared):
    """Queries of one head that look for one key: the first tokens, keys far
    back, at page and tile borders and next to them.  The key carries most of
    the weight, so a missing or misplaced one cannot hide."""
    layer = cases.attention(4, 2, 32, 24, 1.2)
    layers = [layer]
    if shared:
        layers = [layer, cases.attention(4, 2, 32, 24, 1.2, kv_from=0)]
    m = Mixer(layers, 160, dtype, device)
    w = {k: v.double() for k, v in m.w.items()}
    T, head, pre = 700, 2, f"l{len(layers) - 1}.mix."
    g = torch.Generator().manual_seed(5)
    h = torch.randn(T, 160, generator=g, dtype=torch.float64)
    asks = {40: 31, 41: 32, 66: 63, 67: 64, 100: 0, 140: 126, 129: 127, 130: 128, 191: 127,
            192: 15, 193: 16, 259: 31, 258: 47, 300: 1, 319: 255, 320: 256, 321: 257, 400: 383,
            449: 384, 500: 2, 640: 575, 641: 576, 698: 0, 699: 697}
    heads = lambda x, layer, n: oracle.rms(  # noqa: E731
        (x @ w[f"{layer}{n}"].T).view(len(x), -1, 32), m.eps) * w[f"{layer}{n}.norm"]
    for q, k in asks.items():
        key = heads(h[k: k + 1], "l0.mix.", "k")[0, head // 2] / w[pre + "q.norm"]
        want = torch.randn(128, dtype=torch.float64, generator=g)
        want[head * 32: (head + 1) * 32] = key
        h[q] = torch.linalg.lstsq(w[pre + "q"], want[:, None]).solution[:, 0] * 3
    h = h.to(dtype).double()
    qs, ks = heads(h, pre, "q"), heads(h, "l0.mix.", "k")
    for q, k in asks.items():
        s = ks[: q + 1, head // 2] @ qs[q, head] * 1.2
        s = torch.cat([s, w[pre + "sink"][head: head + 1]])
        assert torch.softmax(s, 0)[k] > 0.5, (q, k)
    want, rows = m.want(h), sorted(asks)
    tol = 3e-5 if dtype == F32 else 5e-2
    for sizes in ([T], [90, 1], [T - 70, 1], [128, 128, 2], [97, 3], [16], [63, 2, 65]):
        got = m.run(h, sizes)
        assert cases.error(got[rows], want[rows]) < tol, sizes


DELTAS = {
    "plain": cases.delta(4, 2, 24, 40, 4),
    "own keys": cases.delta(3, 3, 32, 16, 3, (16, 16)),
    "one": cases.delta(1, 1, 1, 1, 1, (1, 1)),
    "shared keys": cases.delta(8, 1, 16, 32, 4, (4, 24)),
    "odd": cases.delta(3, 1, 33, 17, 2, (5, 3)),
    "64/48": cases.delta(4, 2, 64, 48, 3),
    "128": cases.delta(2, 2, 128, 128, 4, (32, 32)),
    "100/50": cases.delta(2, 1, 100, 50, 5),
    "deep": cases.delta(2, 1, 200, 24, 8),
    "long rows": cases.delta(1, 1, 24, 300, 4),
    "deepest": cases.delta(1, 1, 512, 64, 2),
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", DELTAS)
def test_delta(device, dtype, kind):
    m = Mixer(DELTAS[kind], 64, dtype, device, eps=1e-3)
    h = torch.randn(3 * CHUNK + 11, 64, generator=torch.Generator().manual_seed(3))
    want = m.want(h)
    T = len(h)
    tol = 3e-5 if dtype == F32 else 8e-2
    for sizes in ([T], [1], [CHUNK, 17, 2, 60], [16], [2, 3, 129], [CHUNK + 1, 15, 16]):
        got = m.run(h, sizes)
        e = cases.row_errors(got, want)
        assert float(e.quantile(0.95)) < tol and float(e.max()) < 4 * tol, sizes


def delta_request(sh, z, beta, dtype, device, sizes, q, k, v):
    """The recurrence alone: no convolution, rows given as they enter silu, the
    output gate wide open and its norm with weight one."""
    T, H, V = len(z), sh.heads, sh.vdim
    state = PagedState([StateSpec(
        H, sh.dim, V, sh.channels, 0)], T, 1, dtype, device)
    cases.poison(state)
    held = state.admit("x")
    state.reserve("x", T)
    y = torch.zeros(T, -(-(sh.columns[5] + H) // 8) * 8)
    for at, t in zip(sh.places[:3], (q, k, v)):
        y[:, at: at + t[0].numel()] = t.reshape(T, -1)
    y[:, sh.places[5]: sh.places[5] + H] = beta
    y, z = y.to(device, dtype), z.to(device, dtype)
    ones = lambda *s: torch.ones(*s, device=device, dtype=dtype)  # noqa: E731
    zeros = lambda *s: torch.zeros(*s, device=device, dtype=dtype)  # noqa: E731
    outs, at = [], 0
    for n in cases.cut(T, sizes):
        out = ragged.gated_delta(
            y[at: at + n], ones(sh.channels, 1), zeros(H), zeros(H * sh.dim), ones(V),
            state.layers[0], sh, 1e-6, RaggedBatch([(held, n)], device), z[at: at + n], True)
        outs.append(out.cpu())
        at += n
        held.length = at
    return torch.cat(outs)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("case", ["mixed", "cliffs", "keeps", "forgets"])
@pytest.mark.parametrize("D", [16, 24, 64, 160])
def test_decays_per_channel(device, case, D):
    """Decays that differ by orders of magnitude between channels and from token
    to token: hard ones beside ones that keep everything must not spoil each
    other (no overflow, no lost digits), over chunk borders and in portions."""
    H, KH, V, T = 4, 2, 24, 2 * CHUNK + 40
    sh = DeltaShape(H, KH, D, V, 1, (1, 1))
    g = torch.Generator().manual_seed(6)
    q, k = (torch.randn(T, KH, D, generator=g) for _ in "qk")
    v = torch.randn(T, H, V, generator=g)
    beta = torch.randn(T, H, generator=g)
    a = torch.randn(T, H, D, generator=g)
    if case == "mixed":
        a = torch.linspace(-12, 60, D).expand(T, H, D) + a
    elif case == "cliffs":       # almost all kept, now and then almost all lost
        a = torch.where(torch.rand(T, H, D, generator=g) < 0.1, 90.0, -14.0)
    elif case == "keeps":
        a = a - 16
    else:
        a = a + 30
    z = torch.cat([a.reshape(T, -1), torch.full((T, H * V), 40.0)], 1)
    d = lambda t: t.double()  # noqa: E731
    idx = [h // 2 for h in range(H)]
    qn = (oracle.unit(oracle.silu(d(q))) * D ** -0.5)[:, idx]
    kn = oracle.unit(oracle.silu(d(k)))[:, idx]
    o = oracle.delta_rule(qn, kn, oracle.silu(d(v)), oracle.sigmoid(d(beta)),
                          torch.exp(-oracle.softplus(d(a))))
    want = oracle.rms(o, 1e-6).reshape(T, -1)
    for sizes in ([T], [1], [CHUNK - 1, 2, CHUNK + 3, 1], [16], [70, 17]):
        got = delta_request(sh, z, beta, F32, device, sizes, q, k, v)
        assert cases.error(got, want) < 1e-4, sizes


@pytest.mark.parametrize("device", DEVICES)
def test_delta_remembers(device):
    """One write, read out long after through the one channel that keeps; what
    was lost at a chunk's, a block's or a portion's border would show."""
    H, D, V, T = 1, 32, 16, 4 * CHUNK + 5
    sh = DeltaShape(H, 1, D, V, 1, (1, 1))
    keep = 19
    for at in (0, 15, 16, 33, 62, 63, 64, 100, CHUNK + 47):
        q = torch.full((T, 1, D), -60.0)     # silu of it is nothing
        k, v = q.clone(), torch.zeros(T, 1, V)
        q[:, 0, keep] = 3.0
        k[at, 0, keep] = 3.0
        v[at, 0] = torch.arange(1, V + 1).float()
        a = torch.full((T, H, D), 50.0)
        a[..., keep] = -40.0
        z = torch.cat([a.reshape(T, -1), torch.full((T, H * V), 40.0)], 1)
        beta = torch.full((T, H), 40.0)
        row = oracle.rms(oracle.silu(v[at, 0].double()), 1e-6)
        for sizes in ([T], [at + 1, T], [1] * (at + 1) + [T], [70, 1], [16]):
            got = delta_request(sh, z, beta, F32, device, sizes, q, k, v).double()
            assert float(got[:at].abs().max()) < 1e-3 if at else True
            assert float((got[at:] - row).abs().max()) < 1e-3, (at, sizes)


@pytest.mark.parametrize("device", DEVICES)
def test_future_is_not_seen(device):
    """A loud token at i + 1 does not change what token i gives."""
    for layer in (cases.attention(4, 2, 32, 16), cases.delta(4, 2, 16, 24, 4)):
        m = Mixer(layer, 64, F32, device)
        h = torch.randn(150, 64, generator=torch.Generator().manual_seed(3))
        base = m.run(h, [150])
        for i in (0, 15, 16, 31, 62, 63, 64, 127, 128):
            loud = h.clone()
            loud[i + 1:] = 50 * torch.randn(149 - i, 64)
            assert cases.error(m.run(loud, [150])[: i + 1], base[: i + 1]) < 1e-6, i


def test_other_combinations():
    """The pieces are usable apart, and refuse what they cannot be."""
    for bad in (dict(qk_norm=True, head_weights=True), dict(qk_norm=True, head_norm=True)):
        with pytest.raises(ValueError):
            GroupedAttention(32, 4, 2, 16, 8, 0.25, 1e-5, **bad)
    with pytest.raises(ValueError):
        GatedDelta(32, 4, 3, 8, 8, 4, 1e-5)
    with pytest.raises(ValueError):
        GatedDelta(32, 4, 2, 8, 8, 4, 1e-5, gate="tanh")
    with pytest.raises(ValueError):
        Routing("linear")
    m = RoutedExperts(32, 8, 4, 2, 2, F32, routing=Routing(on_input=True))
    with pytest.raises(ValueError):
        m.rows(torch.zeros(1, 64))
    with pytest.raises(ValueError):
        m(torch.zeros(1, 32), torch.zeros(1, 64))
    # a delta rule with low-rank decay and a silu gate
    g = torch.Generator().manual_seed(1)
    m = GatedDelta(32, 2, 1, 8, 8, 3, 1e-5, F32, ranks=(3, 5))
    for p in m.parameters():
        p.data = torch.randn(p.shape, generator=g) * 0.4
    state = PagedState([m.store_spec()], 64, 1, F32, "cpu")
    held = state.admit(0)
    state.reserve(0, 30)
    h = torch.randn(30, 32, generator=g)
    got = m(h, RaggedBatch([(held, 30)], "cpu"), state.layers[0])
    # the oracle's gate is a sigmoid; silu(x) = x sigmoid(x)
    w = {f"m.{k.replace('.weight', '')}": v for k, v in m.state_dict().items()}
    x = (h @ w["m.g1"].T) @ w["m.g2"].T
    w["m.o"], o = torch.eye(16), w["m.o"]
    want = (oracle.channel_delta(h, w, "m.", {"heads": 2, "kv_heads": 1, "dim": 8, "vdim": 8},
                                 1e-5) * x) @ o.T
    assert cases.error(got, want) < 1e-5


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
    toks = cases.tokens(cfg, 80)
    want = cases.expected("mixed", toks)

    def off(change=lambda t: None, edit=lambda c: None):
        other, c = {k: v.clone() for k, v in w.items()}, copy.deepcopy(cfg)
        change(other)
        edit(c)
        return cases.error(oracle.forward(c, other, toks), want)

    assert off() == 0
    for i, layer in enumerate(cfg["layers"]):
        names = ["norm1"]
        if layer["type"] == "attention":
            names += ["mix.q.norm", "mix.sink", "mix.g"]
            if "kv_from" not in layer["mixer"]:
                names += ["mix.k.norm", "mix.v"]
        else:
            names += ["mix.q.conv", "mix.v.conv", "mix.b", "mix.a1", "mix.a2", "mix.g2",
                      "mix.A_log", "mix.dt_bias", "mix.norm"]
        if layer["mlp"] is not None:
            names += ["norm2", "mlp.gate.b", "mlp.up.b", "mlp.down.b"] \
                if layer["mlp"]["kind"] == "dense" else ["norm2", "mlp.router", "mlp.e0.gate"]
        for n in names:
            def change(t, key=f"l{i}.{n}"):
                t[key] = torch.zeros_like(t[key])
            assert off(change) > 0.005, (i, n)
    for edit in (lambda c: c["embedding"].update(scale=1.3),
                 lambda c: c["norm"].update(eps=0.1),
                 lambda c: c["layers"][2]["mixer"].update(scale=0.5),
                 lambda c: c["layers"][2]["mixer"].update(kv_from=5),
                 lambda c: c["layers"][0]["mlp"]["expert"].update(limit=1.0),
                 lambda c: c["layers"][4]["mlp"].update(limit=1.0),
                 lambda c: c["layers"][0]["mlp"]["router"].update(top=2)):
        try:
            assert off(edit=edit) > 0.005
        except KeyError:        # a source that has not run yet
            pass


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
    """The start of a sequence: convolutions and states begin with nothing, and
    the first token sees itself and the sink."""
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
    """Many chunks and pages, whole and cut."""
    toks = cases.tokens(cases.CONFIGS["mixed"], 700, 9)
    want = cases.expected("mixed", toks)
    e = engine("mixed", device, F32, max_tokens=768)
    for sizes in ([700], [300, 129, 2, 269], [CHUNK]):
        got = cases.replay(e, {"r": toks}, [[("r", n)] for n in cases.cut(700, sizes)])
        assert cases.model_error(got["r"], want, F32) < 1, sizes


@pytest.mark.gpu
def test_kernels_refuse_bad_operands():
    ext = ragged.hip_ragged()
    assert ext is not None
    dev = dict(device="cuda")
    _, batch = batch_of({"a": (0, 20)}, "cuda")
    x, w = torch.zeros(20, 64, **dev), torch.ones(64, **dev)
    where = torch.zeros(20, 2, dtype=torch.int32, **dev)
    norm = lambda y, where, wide: ext.add_norm(  # noqa: E731
        x, y, w, None, True, 1e-6, 0.0, 1.0, where, wide)
    q, pool, out = (torch.zeros(*s, **dev) for s in ((20, 4, 32), (640, 96), (20, 64)))
    attn = lambda gate: ext.grouped_attn_short(  # noqa: E731
        q, None, pool, out, batch.cu, batch.pos0, batch.pages, 1, 20, 20, 20, 2, 16, 16, 1.0, 0,
        None, None, batch.tok_pos, gate)
    y = torch.zeros(20, 224, **dev)
    turn = lambda y, w, norm, own: ext.grouped_turn(  # noqa: E731
        y, w, None, 1e-6, norm, None, None, None, None, pool, 4, 2, 32, 16, 32, 16,
        batch.tok_pos, batch.tok_entry, batch.pages, 20, own)
    sh = DeltaShape(2, 1, 16, 8, 1, (8, 8))
    rows, z = torch.zeros(20, 80, **dev), torch.zeros(20, 48, **dev)
    delta = lambda z, dt: ext.delta_short(  # noqa: E731
        rows[:4], torch.ones(48, 1, **dev), torch.zeros(2, **dev), torch.zeros(dt, **dev),
        torch.ones(8, **dev), torch.zeros(1, 2, 16, 8, **dev), torch.zeros(1, 48, 0, **dev),
        torch.zeros(4, 16, **dev), torch.tensor([0, 4], dtype=torch.int32, **dev), batch.pos0,
        batch.slots, 1, 4, 1, 2, 16, 8, sh.places, 1e-6, z, True)
    h, tiles = torch.zeros(20, 64, **dev), torch.zeros(4, 3, dtype=torch.int32, **dev)
    gemm = lambda O, scale: ext.expert_gemm(  # noqa: E731
        h, None, tiles, torch.zeros(3, O, 64, **dev), scale, 16, 20, 2, 1.0, 1.702)
    norm(x.clone(), None, 64), attn(torch.zeros(20, 4, **dev)), delta(z[:4], 32)
    turn(y, w[:32], True, True), turn(y[:, :128], w[:32], True, False), gemm(64, None)
    torch.cuda.synchronize()
    for i, call in enumerate((
            lambda: norm(x.clone(), where, 64), lambda: norm(x.clone(), None, 32),
            lambda: norm(x.bfloat16(), None, 64), lambda: attn(torch.zeros(20, 2, **dev)),
            lambda: attn(torch.zeros(10, 4, **dev)), lambda: turn(y[:, :128], w[:32], True, True),
            lambda: turn(y, w, True, True), lambda: turn(y, w[:32], False, True),
            lambda: delta(z, 32), lambda: delta(z[:4, :40], 32), lambda: delta(z[:4], 2),
            lambda: gemm(48, None), lambda: gemm(64, torch.zeros(10, **dev)),
            lambda: ext.clamped_glu(h, h[:, :32], 1.0, 1.702))):
        with pytest.raises(RuntimeError):
            call()
            raise AssertionError(i)


@pytest.mark.gpu
def test_bf16_matches_cpu_path_on_kernel_shapes():
    """The shapes a real model has, GPU kernels against the torch path."""
    g = torch.Generator().manual_seed(9)
    for layer in (cases.attention(16, 4, 128, 128), cases.delta(4, 2, 128, 128, 4, (128, 128))):
        a = Mixer(layer, 256, BF16, "cuda")
        b = Mixer(layer, 256, F32, "cpu", a.w)
        h = torch.randn(1100, 256, generator=g)
        want = b.run(h.bfloat16().float(), [1100])
        for sizes in ([1100], [1000, 1], [300, 128, 16]):
            assert cases.error(a.run(h, sizes), want) < 4e-2
