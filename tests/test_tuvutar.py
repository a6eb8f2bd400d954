"""Tuvutar against the plain oracle: mechanisms alone, then the batch engine."""

import math

import pytest
import torch

import tuvutar_cases as cases
import tuvutar_oracle as oracle
from mlx_sharding_amd.ops import ragged
from mlx_sharding_amd.ops.paged import PagedState, RaggedBatch
from mlx_sharding_amd.ops.ragged import Rotary
from mlx_sharding_amd.parallel.batching import BatchEngine, CacheFull, Portion


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

@pytest.mark.parametrize("scaling", [
    None,
    {"factor": 4.0, "original": 256, "fast": 24.0, "slow": 1.0},
    {"factor": 32.0, "original": 64, "fast": 32.0, "slow": 0.01},   # both clamps
    {"factor": 2.0, "original": 100000, "fast": 1e-3, "slow": 1e-3},
    {"factor": 1.0, "original": 64, "fast": 2.0, "slow": 1.0},
    {"factor": 0.5, "original": 512, "fast": 16.0, "slow": 2.0},
])
def test_rotary_frequencies(scaling):
    rot = {"dims": 24, "base": 3000.0, "scaling": scaling}
    r = Rotary(24, 3000.0, *(scaling[k] for k in ("factor", "original", "fast", "slow"))) \
        if scaling else Rotary(24, 3000.0)
    f, m = oracle.rotary_frequencies(rot)
    assert torch.allclose(r.frequencies(), torch.tensor(f, dtype=torch.float64), rtol=1e-12)
    assert r.magnitude == pytest.approx(m)
    cos, sin = r.tables(700, "cpu")
    assert abs(float(cos[699, 3]) - math.cos(699 * f[3]) * m) < 1e-6
    assert abs(float(sin[699, 0]) - math.sin(699 * f[0]) * m) < 1e-6


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [40, 97, 1024, 2500, 9000])
def test_add_norm(device, dtype, W):
    torch.manual_seed(0)
    x = torch.randn(5, W)
    y = (torch.randn(5, W) * 3).to(dtype)
    wp, wn = (torch.randn(W) * 0.3).to(dtype), (torch.randn(W) * 0.3).to(dtype)
    eps = 0.05  # large, so that a misplaced eps shows
    want_x = x.double() + oracle.norm_around_zero(y.double(), wp.double(), eps)
    want_h = oracle.norm_around_zero(want_x, wn.double(), eps)
    xd = x.clone().to(device)
    h = ragged.add_norm(xd, y.to(device), wp.to(device), wn.to(device), eps, 1.0, dtype)
    assert h.dtype == dtype
    assert cases.error(xd, want_x) < 1e-6
    assert cases.error(h, want_h) < (1e-6 if dtype == F32 else 4e-3)
    # either half alone
    xd = x.clone().to(device)
    h = ragged.add_norm(xd, None, None, wn.to(device), eps, 1.0, dtype)
    assert torch.equal(xd.cpu(), x)
    assert cases.error(h, oracle.norm_around_zero(x.double(), wn.double(), eps)) < 4e-3
    assert ragged.add_norm(xd, y.to(device), wp.to(device), None, eps, 1.0, dtype) is None
    assert cases.error(xd, want_x) < 1e-6


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff", [64, 33])
def test_gated_mlp(device, dtype, ff):
    from mlx_sharding_amd.models.mixers import GatedMLP
    torch.manual_seed(0)
    w = {f"m.{n}": (torch.randn(s) * s[1] ** -0.5).to(dtype) for n, s in
         (("gate", (ff, 48)), ("up", (ff, 48)), ("down", (48, ff)))}
    m = GatedMLP(48, ff, "gelu_tanh", dtype)
    m.load_state_dict({k[2:] + ".weight": v for k, v in w.items()})
    m.to(device).prepare()
    h = (torch.randn(7, 48) * 2).to(dtype)
    want = oracle.dense_mlp(h.double(), {k: v.double() for k, v in w.items()}, "m.")
    assert cases.error(m(h.to(device)), want) < (2e-6 if dtype == F32 else 2e-2)


class Mixer:
    """One mixer of a layer with its storage: feed portions, compare."""

    def __init__(self, layer, width, dtype, device, w=None, seed=0, eps=1e-5):
        cfg = cases.config(width, 8, [layer], eps)
        self.w = w or cases.weights(cfg, seed)
        self.model = cases.build(cfg, self.w, device, dtype)
        self.mix = self.model.l0.mix
        self.layer, self.dtype, self.device, self.eps = layer, dtype, device, eps

    def want(self, h):
        w = {k: v.double() for k, v in self.w.items()}
        mx, h = self.layer["mixer"], h.to(self.dtype).double()
        if self.layer["type"] == "delta":
            return oracle.delta(h, w, "l0.mix.", mx, self.eps)
        c, kr = oracle.latent_rows(h, w, "l0.mix.", mx, self.eps)
        return oracle.latent_attention(h, w, "l0.mix.", mx, c, kr)

    def run(self, h, sizes):
        """h [T, width] in portions of these sizes (the last one repeated)."""
        T = h.shape[0]
        state = self.model.make_state(T + 64, 2)
        cases.poison(state)
        state.admit("other")       # so that slot and pages are not the first
        state.reserve("other", 1)
        held = state.admit("x")
        outs, at = [], 0
        for n in cases.cut(T, sizes):
            state.reserve("x", at + n)
            batch = RaggedBatch([(held, n)], self.device)
            hp = h[at: at + n].to(self.device, self.dtype)
            if self.layer["type"] == "delta":
                y = self.mix(hp, batch, state.layers[0])
            else:
                y = self.mix(hp, batch, state.layers[0], self.model._rotation(
                    self.mix.rotary, batch.max_pos, hp.device))
            outs.append(y.cpu())
            at += n
            held.length = at
        return torch.cat(outs)


LATENTS = {
    "plain": cases.latent(3, 24, 16, 40, 48),
    "yarn": cases.latent(4, 32, 32, 64, 64, scaling=cases.YARN),
    "one": cases.latent(1, 8, 2, 8, 8),
    "wide": cases.latent(16, 128, 64, 128, 512),
    "many": cases.latent(20, 16, 8, 16, 96),
    "too wide to expand": cases.latent(2, 240, 32, 272, 40),
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", LATENTS)
def test_latent_attention(device, dtype, kind):
    m = Mixer(LATENTS[kind], 64, dtype, device)
    h = torch.randn(150, 64, generator=torch.Generator().manual_seed(3))
    want = m.want(h)
    tol = 2e-5 if dtype == F32 else 3e-2
    for sizes in ([150], [1], [64, 17, 2, 60], [16], [2, 3, 129]):
        assert cases.error(m.run(h, sizes), want) < tol, sizes


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_latent_single_key_stands_out(device, dtype):
    """Queries that look for one key far back, at page and tile borders: the
    key carries more than half of the weight, so a missing or misplaced one
    cannot hide among hundreds."""
    layer = cases.latent(2, 64, 8, 24, 96)
    mx = layer["mixer"]
    m = Mixer(layer, 128, dtype, device)
    w = {k: v.double() for k, v in m.w.items()}
    g = torch.Generator().manual_seed(5)
    T = 330
    h = torch.randn(T, 128, generator=g, dtype=torch.float64)
    asks = {100: 0, 128: 63, 131: 64, 191: 127, 192: 128, 255: 31, 256: 32,
            260: 260, 300: 1, 319: 255, 320: 256, 322: 322, 329: 0}
    wq = w["l0.mix.q"].reshape(2, 72, 128)[0]
    for q, k in asks.items():
        if q == k:
            continue
        c, kr = oracle.latent_rows(h[: k + 1], w, "l0.mix.", mx, m.eps)
        key = (w["l0.mix.uk"].reshape(2, 64, 96)[0] @ c[k])
        want = torch.cat([key, torch.zeros(8, dtype=torch.float64)])
        d = torch.linalg.lstsq(wq, want[:, None]).solution[:, 0]
        h[q] = 18.0 * d / (key @ key * mx["scale"])
    h = h.to(dtype).double()
    c, kr = oracle.latent_rows(h, w, "l0.mix.", mx, m.eps)
    for q, k in asks.items():
        if q == k:
            continue
        qv = wq @ h[q]
        keys = c[: q + 1] @ w["l0.mix.uk"].reshape(2, 64, 96)[0].T
        s = (keys @ qv[:64] + kr[: q + 1] @ oracle.rotate(
            qv[64:].expand(q + 1, 8).contiguous(), mx["rot"])[q]) * mx["scale"]
        assert torch.softmax(s, 0)[k] > 0.5, (q, k)
    want = m.want(h)
    tol = 2e-4 if dtype == F32 else 8e-2
    for sizes in ([T], [90, 1], [T - 40, 1], [128, 128, 2], [97, 3]):
        got = m.run(h, sizes)
        rows = sorted(asks)
        assert cases.error(got[rows], want[rows]) < tol, sizes


DELTAS = {
    "grouped": cases.delta(6, 2, 20, 36, 3),
    "equal": cases.delta(2, 2, 32, 32, 4),
    "one": cases.delta(1, 1, 4, 4, 1),
    "long taps": cases.delta(4, 4, 33, 17, 8),
    "real": cases.delta(4, 2, 128, 128, 4),
    "deep": cases.delta(2, 1, 200, 16, 2),
    "flat": cases.delta(2, 1, 8, 300, 4),
    "big": cases.delta(1, 1, 256, 256, 4),
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", DELTAS)
def test_gated_delta(device, dtype, kind):
    m = Mixer(DELTAS[kind], 48, dtype, device)
    h = torch.randn(150, 48, generator=torch.Generator().manual_seed(3))
    want = m.want(h)
    tol = 5e-5 if dtype == F32 else 5e-2
    for sizes in ([150], [1], [64, 17, 2, 67], [16], [2, 3, 129], [63, 65, 1]):
        assert cases.error(m.run(h, sizes), want) < tol, sizes


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("A_log,dt,note", [
    (-12.0, -3.0, "nothing is forgotten"),
    (4.0, 2.0, "all is forgotten at once"),
    (1.0, None, "strong and weak decays alternate"),
])
def test_gated_delta_decays(device, A_log, dt, note):
    layer = cases.delta(2, 1, 16, 16, 4)
    w = cases.weights(cases.config(48, 8, [layer]), 0)
    w["l0.mix.A_log"] = torch.full((2,), A_log).bfloat16()
    if dt is None:  # softplus arguments around +-30
        w["l0.mix.a"] = w["l0.mix.a"] * 20
    else:
        w["l0.mix.dt_bias"] = torch.full((2,), dt).bfloat16()
    m = Mixer(layer, 48, F32, device, w)
    h = torch.randn(200, 48, generator=torch.Generator().manual_seed(4))
    want = m.want(h)
    for sizes in ([200], [1], [70, 130]):
        # rows whose output is nearly nothing are normed up, with their noise
        assert cases.error(m.run(h, sizes), want) < 2e-3, (note, sizes)


@pytest.mark.parametrize("device", DEVICES)
def test_gated_delta_remembers_one_write(device):
    """One strong write at the first token, at chunk borders and next to them,
    read back by a query of the same direction hundreds of tokens later."""
    layer = cases.delta(1, 1, 16, 16, 2)
    w = cases.weights(cases.config(48, 8, [layer]), 0)
    w["l0.mix.A_log"] = torch.tensor([-9.0]).bfloat16()
    for n in ("q", "k"):
        w[f"l0.mix.{n}"] = w["l0.mix.q"]
        w[f"l0.mix.{n}.conv"] = torch.tensor([0.0, 1.0]).repeat(16, 1).bfloat16()
    m = Mixer(layer, 48, F32, device, w)
    g = torch.Generator().manual_seed(6)
    # directions that q and k do not see: the reader's own value is another,
    # and beta can be set: strong for the write, next to nothing in between
    unseen = torch.linalg.svd(w["l0.mix.q"].float()).Vh[16:]
    wb = w["l0.mix.b"].float()[0]

    def with_beta(x, logit):
        d = unseen.T @ (unseen @ wb)
        return x + d * (logit - x @ wb) / (d @ wb)

    for place in (0, 1, 15, 16, 62, 63, 64, 65, 127, 128):
        h = torch.stack([with_beta(x, -14.0)
                         for x in torch.randn(200, 48, generator=g)])
        loud = torch.randn(48, generator=g) * 3
        h[place] = with_beta(loud, 4.0)
        h[199] = with_beta(loud + 3 * torch.randn(32, generator=g) @ unseen, -2.0)
        want = m.want(h)
        quiet = h.clone()
        quiet[place] = with_beta(quiet[place], -14.0)
        assert cases.error(m.want(quiet)[199:], want[199:]) > 0.02
        for sizes in ([200], [place + 1, 1], [199, 1], [64, 2, 70]):
            assert cases.error(m.run(h, sizes)[199:], want[199:]) < 1e-4, (place, sizes)


# ---------------------------------------------------------------------------
# The engine: whole models, portions, batches, pages and slots
# ---------------------------------------------------------------------------

def engine(name, device, dtype, max_tokens=512, max_requests=4, seed=0):
    cfg = cases.CONFIGS[name]
    e = BatchEngine(cases.build(cfg, cases.weights(cfg, seed), device, dtype),
                    max_tokens, max_requests)
    cases.poison(e.state)
    return e


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
def test_unequal_batch(device, dtype):
    """Portions of prompts beside single tokens; requests pause, end, and
    others take over their pages and slots."""
    cfg = cases.CONFIGS["mixed"]
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
    e = engine("mixed", device, dtype, max_tokens=448)
    got = cases.replay(e, streams, schedule)
    for r, toks in streams.items():
        n = sum(k for step in schedule for q, k in step if q == r)
        want = cases.expected("mixed", toks)[:n]
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
@pytest.mark.parametrize("n", [1, 2, 3, 4, 5])
def test_first_tokens(device, dtype, n):
    """The start of a sequence, shorter than the convolutions."""
    toks = cases.tokens(cases.CONFIGS["mixed"], n, 7)
    want = cases.expected("mixed", toks)
    for sizes in ([n], [1], [2, 1]):
        e = engine("mixed", device, dtype)
        got = cases.replay(e, {"r": toks}, [[("r", k)] for k in cases.cut(n, sizes)])
        assert cases.model_error(got["r"], want, dtype) < 1


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding(device):
    toks = cases.tokens(cases.CONFIGS["mixed"], 330, 8)
    want = cases.expected("mixed", toks)
    e = engine("mixed", device, F32)
    got = cases.replay(e, {"r": toks}, [[("r", 5)]] + [[("r", 1)]] * 325)
    assert cases.model_error(got["r"], want, F32) < 1


def test_engine_refuses_cleanly():
    e = engine("ones", "cpu", F32, max_tokens=128, max_requests=2)
    e.step([Portion("a", [1, 2], [])])
    with pytest.raises(CacheFull):      # pages
        e.step([Portion("b", [1] * 65), Portion("a", [3])])
    assert e.live == ["a"] and e.length("a") == 2 and e.state.free_slots == 1
    e.step([Portion("b", [1])])
    with pytest.raises(CacheFull):      # slots
        e.step([Portion("c", [1])])
    for bad in ([Portion("a", [])], [Portion("a", [67])], [Portion("a", [-1])],
                [Portion("a", [1], [1])], [Portion("a", [1]), Portion("a", [2])]):
        with pytest.raises(ValueError):
            e.step(bad)
    toks = [1, 2, 3, 4]
    got = e.step([Portion("a", toks[2:], [0, 1])])
    assert cases.model_error(got, cases.expected("ones", toks)[2:], F32) < 1
    assert e.step([]).shape == (0, 67)


def test_state_manager_bookkeeping():
    s = PagedState([None], 256, 3, F32, "cpu")
    for r in "ab":
        s.admit(r)
    s.reserve("a", 65)
    s.reserve("b", 64)
    assert len(s.live["a"].pages) == 2 and len(s.live["b"].pages) == 1
    with pytest.raises(CacheFull):
        s.reserve("b", 193)
    assert len(s.live["b"].pages) == 1
    with pytest.raises(ValueError):
        s.admit("a")
    mine = set(s.live["a"].pages)
    s.release("a")
    s.grow(6)
    s.reserve("b", 384)
    assert mine < set(s.live["b"].pages) and s.free_tokens == 0
    assert sorted(s.live["b"].pages) == list(range(6))


@pytest.mark.gpu
def test_kernels_refuse_bad_operands():
    ext = ragged.hip_ragged()
    assert ext is not None
    x = torch.randn(4, 64, device="cuda")
    w = torch.randn(64, device="cuda")
    with pytest.raises(RuntimeError):
        ext.add_norm(x, x.bfloat16(), w, w, True, 1e-6, 1.0, 1.0, None, 64)
    with pytest.raises(RuntimeError):
        ext.add_norm(x, None, None, w[:32], True, 1e-6, 1.0, 1.0, None, 64)
    with pytest.raises(RuntimeError):
        ext.latent_gather(torch.zeros(100, 64, device="cuda"),
                          torch.zeros(1, 3, device="cuda", dtype=torch.int32), 64)


@pytest.mark.gpu
def test_bf16_matches_cpu_path_on_kernel_shapes():
    """The shapes a real model has, GPU kernels against the torch path."""
    layer = cases.latent(16, 128, 64, 128, 512, scaling=cases.YARN)
    g = Mixer(layer, 256, BF16, "cuda")
    c = Mixer(layer, 256, F32, "cpu", g.w)
    h = torch.randn(700, 256, generator=torch.Generator().manual_seed(9))
    want = c.run(h.bfloat16().float(), [700])
    for sizes in ([700], [500, 1], [300, 128, 16]):
        assert cases.error(g.run(h, sizes), want) < 3e-2
