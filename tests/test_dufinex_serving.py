"""Dufinex through the framework's entry points: registry and loading,
generation, scheduler and service, pipeline stages, captured decode, replay."""

import io
import json
import os
import socket
import threading

import numpy as np
import pytest
import torch
import torch.multiprocessing as mp

import dufinex_cases as cases
import dufinex_oracle as oracle
from mlx_sharding_amd.config import ModelConfig
from mlx_sharding_amd.models import get_model_class
from mlx_sharding_amd.parallel.batching import (BatchEngine, BatchScheduler,
                                                BatchService, CacheFull)
from mlx_sharding_amd.parallel.engine import (LocalChain, SamplingParams,
                                              generate_step, stream_generate)
from mlx_sharding_amd.utils.loading import load_model, save_sharded_weights

GPU = pytest.param("cuda", marks=pytest.mark.gpu)
DEVICES = ["cpu", GPU]
F32, BF16 = torch.float32, torch.bfloat16
NAME = "stages"
CFG = cases.CONFIGS[NAME]


@pytest.fixture(autouse=True)
def one_thread():
    n = torch.get_num_threads()
    torch.set_num_threads(1)
    yield
    torch.set_num_threads(n)


@pytest.fixture
def checkpoint(tmp_path):
    return cases.write(tmp_path / "ckpt", CFG, cases.weights(CFG))


_GREEDY = {}


def greedy(prompt, n):
    """Greedy continuation by the oracle."""
    key = (tuple(prompt), n)
    if key not in _GREEDY:
        toks = list(prompt)
        w = {k: v.double() for k, v in cases.weights(CFG).items()}
        for _ in range(n):
            toks.append(int(oracle.forward(CFG, w, toks)[-1].argmax()))
        _GREEDY[key] = toks[len(prompt):]
    return _GREEDY[key]


def model(device="cpu", dtype=F32, **kw):
    return cases.build(CFG, cases.weights(CFG), device, dtype, **kw)


# ---------------------------------------------------------------------------
# Registry, configuration, weights
# ---------------------------------------------------------------------------

def test_config_and_registry():
    cls = get_model_class("dufinex")
    c = ranked()
    assert (c.model_type, c.num_hidden_layers, c.hidden_size, c.vocab_size) == \
        ("dufinex", 5, 96, 131)
    assert cls.supports_ragged and cls.allowed_cuts(c) == [1, 3, 4]
    cls(c, c.shard())
    for change in (lambda r: r["layers"][0].update(type="other"),
                   lambda r: r["layers"][0]["mlp"].update(kind="other"),
                   lambda r: r["layers"][2]["mlp"]["router"].update(top=6),
                   lambda r: r["layers"][1]["mixer"].update(kv_heads=3),
                   lambda r: r["layers"][0]["mixer"].update(kv_heads=4),
                   lambda r: r["layers"][1]["mixer"].update(dim=513),
                   lambda r: r["layers"][2]["mixer"].update(dim=16),     # unlike its source
                   lambda r: r["layers"][2]["mixer"].update(heads=2),
                   lambda r: r["layers"][2]["mixer"].update(kv_from=0),  # keeps a state
                   lambda r: r["layers"][2]["mixer"].update(kv_from=2),
                   lambda r: r["layers"][2]["mixer"].update(kv_from=4),
                   lambda r: (r["layers"][4].update(mixer=dict(r["layers"][2]["mixer"], kv_from=2)))):
        bad = json.loads(json.dumps(c.raw))
        change(bad)
        with pytest.raises(ValueError):
            cls(ModelConfig.from_dict(bad), c.shard())
    for cut in (1, 3, 4):
        cls(c, c.shard(0, cut)), cls(c, c.shard(cut, 5))
    with pytest.raises(ValueError):
        cls(c, c.shard(2, 5))


def ranked():
    """The configuration with what its tensors tell besides."""
    c = ModelConfig.from_dict(json.loads(json.dumps(CFG)))
    get_model_class("dufinex").complete_config(c, cases.weights(CFG))
    return c


def test_ranks_come_from_the_tensors():
    c = ranked()
    assert [(s["mixer"]["decay_rank"], s["mixer"]["gate_rank"]) for s in c["layers"]
            if s["type"] == "channel_delta"] == [(12, 7), (6, 10)]
    assert "decay_rank" not in CFG["layers"][0]["mixer"]


def test_who_has_the_embedding():
    """It makes the logits too, so both ends have it."""
    c, cls = ranked(), get_model_class("dufinex")
    for start, end, has in ((0, 1, True), (1, 3, False), (3, 5, True), (0, 5, True)):
        m = cls(c, c.shard(start, end))
        assert ("embed.weight" in m.state_dict()) == has
        assert "head.weight" not in m.state_dict() and m.hop_width == 96


def test_what_layers_keep():
    state = model().make_state(128, 3)
    assert [s is not None for s in state.layers] == [True, True, False, True, True]
    assert state.layers[0].state.shape == (3, 6, 20, 36)
    assert state.layers[0].conv.shape == (3, 2 * 40 + 216, 2)
    assert state.layers[1].rows.shape == (128, 2 * (32 + 16))


@pytest.mark.parametrize("name", ["dufinex-7b", "debug-dufinex"])
def test_presets(name):
    from mlx_sharding_amd.utils.presets import get_preset
    c = get_preset(name)
    assert c.model_type == "dufinex"
    if name.startswith("debug"):
        m = get_model_class("dufinex")(c, c.shard())
        assert {type(m.layer(i).mix).__name__ for i in range(c.num_hidden_layers)} == \
            {"GroupedAttention", "GatedDelta"}


@pytest.mark.parametrize("device", DEVICES)
def test_load_model(checkpoint, device):
    toks = cases.tokens(CFG, 30)
    for dtype in (None, BF16, F32):
        m, c = load_model(checkpoint, device=device, dtype=dtype)
        assert {p.dtype for p in m.parameters()} == {dtype or BF16}
        got = m(torch.tensor([toks], device=device))[0]
        assert got.dtype == F32
        assert cases.model_error(got, cases.expected(NAME, toks), dtype or BF16) < 1
    # a saved state dict loads as well
    m2 = get_model_class("dufinex")(c, c.shard())
    m2.to(F32).load_weights({k: v.clone() for k, v in m.state_dict().items()})
    assert cases.model_error(m2.to(device)(torch.tensor([toks], device=device))[0],
                             cases.expected(NAME, toks), F32) < 1


def test_load_refuses(checkpoint, tmp_path):
    with pytest.raises(ValueError, match="quantized"):
        load_model(checkpoint, quantize=(4, 32))
    for key in ("l1.mix.sink", "l2.mix.g", "l0.mlp.up.b", "l3.mlp.router", "embed", "l4.norm1",
                "l0.mix.q.conv", "l1.mix.k.norm", "l3.mix.b", "l0.mix.g2"):
        w = cases.weights(CFG)
        del w[key]
        with pytest.raises(RuntimeError, match=key):
            load_model(cases.write(tmp_path / key, CFG, w))
    for e in (0, 2, 4):      # an expert in the middle or at an end is missing
        w = cases.weights(CFG)
        del w[f"l2.mlp.e{e}.up"]
        with pytest.raises(RuntimeError, match="l2.mlp"):
            load_model(cases.write(tmp_path / f"e{e}", CFG, w))
    w = cases.weights(CFG)
    w["l4.norm2"] = w["l0.norm2"]   # a layer without a feed-forward
    with pytest.raises(RuntimeError, match="l4.norm2"):
        load_model(cases.write(tmp_path / "extra", CFG, w))


@pytest.mark.parametrize("cut", [1, 3, 4])
def test_split_checkpoint(checkpoint, tmp_path, cut):
    toks = torch.tensor([cases.tokens(CFG, 20)])
    a = save_sharded_weights(checkpoint, tmp_path / "a", 0, cut).parent
    b = save_sharded_weights(checkpoint, tmp_path / "b", cut, 5).parent
    m0, _ = load_model(a, dtype=F32)
    m1, _ = load_model(b, dtype=F32)
    h = m0(toks)
    assert h.dtype == F32 and h.shape == (1, 20, m1.hop_width)
    assert cases.model_error(m1(h)[0], cases.expected(NAME, toks[0].tolist()), F32) < 1


# ---------------------------------------------------------------------------
# Generation
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation(device):
    """stream_generate (the command line's entry point) and the per-request
    loop, against the oracle."""
    prompt = cases.tokens(CFG, 21, 2)
    want = greedy(prompt, 12)
    m = model(device)
    ids = torch.tensor([prompt], device=device)
    assert [t for t, _ in stream_generate(ids, m, max_tokens=12)] == want
    for chunk in (0, 5):
        gen = generate_step(ids, m, m.make_cache(), prefill_chunk=chunk)
        assert [next(gen)[0] for _ in range(12)] == want


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("budget", [2, 7, 24, 512])
def test_scheduler(device, budget):
    """More requests than slots, a small pool, prompts cut by the budget."""
    e = BatchEngine(model(device), 192, 3)
    cases.poison(e.state)
    s = BatchScheduler(e, token_budget=budget)
    prompts = [cases.tokens(CFG, n, 30 + n) for n in (21, 1, 33, 5, 18)]
    reqs = [s.submit(p, max_tokens=6 + i) for i, p in enumerate(prompts)]
    steps = 0
    while s.busy:
        s.step()
        steps += 1
        assert steps < 500
    for i, (r, p) in enumerate(zip(reqs, prompts)):
        assert r.finished and r.output == greedy(p, 6 + i)
    assert e.state.free_tokens == 192 and e.state.free_slots == 3


def test_service_shares_batches():
    svc = BatchService(BatchScheduler(BatchEngine(model(), 512, 3), 16))
    prompts = [cases.tokens(CFG, n, 50 + n) for n in (12, 3, 25, 8)]
    got = [None] * len(prompts)

    def call(i):
        got[i] = [t for t, _ in svc.generate(prompts[i], SamplingParams(max_tokens=7))]

    threads = [threading.Thread(target=call, args=(i,)) for i in range(len(prompts))]
    for t in threads:
        t.start()
    for t in threads:
        t.join(60)
    assert got == [greedy(p, 7) for p in prompts]
    with pytest.raises(CacheFull):
        next(svc.generate([1] * 600, SamplingParams(max_tokens=5)))
    svc.stop()
    assert svc.scheduler.engine.state.free_slots == 3


# ---------------------------------------------------------------------------
# The batch-of-equals cache, stages, pipeline
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("device", DEVICES)
def test_batch_cache(device):
    """forward(x, cache) of the pipeline loops: equal sequences side by side,
    growth beyond the first pages, and reset."""
    m = model(device)
    streams = [cases.tokens(CFG, 90, 60 + i) for i in range(3)]
    x = torch.tensor(streams, device=device)
    cache = m.make_cache(batch_size=3)
    cache[0].shared.GROW = 64

    def feed(sizes, at=0):
        got = []
        for n in sizes:
            got.append(m(x[:, at: at + n], cache).cpu())
            at += n
            assert all(c.offset == at for c in cache)
        return torch.cat(got, 1)

    for _ in range(2):
        for g, s in zip(feed((40, 1, 1, 1, 30, 16, 1)), streams):
            assert cases.model_error(g, cases.expected(NAME, s), F32) < 1
        assert not cache[0].trimmable
        with pytest.raises(ValueError):
            cache[0].trim(50)
        cache[0].trim(0)
        assert cache[3].offset == 0


@pytest.mark.parametrize("cuts", [[1], [1, 3], [4], [1, 3, 4]])
def test_stage_chain(cuts):
    """Stages hand on the residual; same tokens as one."""
    prompt = cases.tokens(CFG, 18, 2)
    ends = [0, *cuts, 5]
    ms = [model(start=a, end=b) for a, b in zip(ends, ends[1:])]
    gen = generate_step(torch.tensor([prompt]), ms[0], ms[0].make_cache(),
                        [LocalChain(m) for m in ms[1:]])
    assert [next(gen)[0] for _ in range(8)] == greedy(prompt, 8)


def test_grpc_stage(checkpoint):
    """A remote stage over the wire gets the 32-bit residual."""
    from mlx_sharding_amd.parallel.grpc_transport import make_clients
    from mlx_sharding_amd.server.shard_server import serve
    prompt = cases.tokens(CFG, 18, 2)
    server, _ = serve(str(checkpoint), 3, 5, dtype=F32, wait=False)
    try:
        remotes = make_clients([f"127.0.0.1:{server._mlxs_port}"])
        m0, _ = load_model(checkpoint, 0, 3, dtype=F32)
        gen = generate_step(torch.tensor([prompt]), m0, m0.make_cache(), remotes)
        assert [next(gen)[0] for _ in range(6)] == greedy(prompt, 8)[:6]
    finally:
        server.stop(0)


def _stage(rank, world, ckpt, port, out_file, prompt, n):
    import torch.distributed as dist

    from mlx_sharding_amd.parallel.rccl import PipelineWorker, split_layers
    torch.set_num_threads(1)
    os.environ.update(MASTER_ADDR="127.0.0.1", MASTER_PORT=str(port))
    dist.init_process_group("gloo", rank=rank, world_size=world)
    c = ModelConfig.load(ckpt)
    s, e = split_layers(c.num_hidden_layers, world,
                        get_model_class(c.model_type).allowed_cuts(c))[rank]
    m, _ = load_model(ckpt, s, e, dtype=F32)
    w = PipelineWorker(m, rank, world, torch.device("cpu"), F32)
    toks = w.prefill([torch.tensor([p]) for p in prompt], 1, len(prompt), len(prompt[0]))
    seq = [[int(t) for t in toks]] if rank == 0 else []
    for _ in range(n - 1):
        toks = w.decode_step(toks, 1, len(prompt))
        if rank == 0:
            seq.append([int(t) for t in toks])
    if rank == 0:
        with open(out_file, "w") as f:
            json.dump(seq, f)
    dist.barrier()
    dist.destroy_process_group()


def test_gloo_pipeline(checkpoint, tmp_path):
    prompts = [cases.tokens(CFG, 18, 2), cases.tokens(CFG, 18, 70)]
    with socket.socket() as s:
        s.bind(("127.0.0.1", 0))
        port = s.getsockname()[1]
    out = str(tmp_path / "tokens.json")
    mp.spawn(_stage, args=(2, str(checkpoint), port, out, prompts, 6), nprocs=2)
    got = json.load(open(out))
    assert list(map(list, zip(*got))) == [greedy(p, 6) for p in prompts]


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_captured_decode(dtype):
    """Graph replays against eager steps, with eager work and waits between;
    twice over the same buffers."""
    from mlx_sharding_amd.parallel.rccl import CapturedDecode, PipelineWorker
    dev = torch.device("cuda", 0)
    m = model("cuda", dtype)
    w = PipelineWorker(m, 0, 1, dev, dtype)
    graph = None
    for seed in (80, 90):
        x = torch.tensor([cases.tokens(CFG, 70, seed + i) for i in range(2)], device=dev)
        ref = m.make_cache(batch_size=2)
        m(x, ref)
        w.prefill([x], 2, 1, 70, return_logits=True, reuse_cache=graph is not None)
        if graph is None:
            graph = CapturedDecode(w, 2, 1, 1024, return_logits=True)
        else:
            assert graph.rearm()
        feed = torch.tensor(cases.tokens(CFG, 20, seed + 5), device=dev)
        for t in range(20):
            tok = feed[t].expand(2, 1).contiguous()
            graph.x_in[0].copy_(tok)
            graph.graphs[0].replay()
            got = graph.tok_out[0].clone()
            if t % 3 == 0:
                torch.cuda.synchronize()
            want = m(tok, ref)[:, -1]
            assert torch.isfinite(got).all()
            assert cases.model_error(got, want, dtype) < 1, t


# ---------------------------------------------------------------------------
# Trace replay
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run(checkpoint, tmp_path, monkeypatch, capsys, device, dtype):
    from mlx_sharding_amd.cli import trace_run
    a, b = cases.tokens(CFG, 40, 11), cases.tokens(CFG, 20, 12)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:19], "want": [18, 0]}], "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": b[:3], "want": []},
                                {"id": "a", "tokens": a[19:20], "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": a[20:], "want": [3]},
                                {"id": "b", "tokens": b[3:5], "want": [0, 1]}],
         "end": ["a"]},
        {"step": 7, "entries": [{"id": "b", "tokens": b[5:], "want": [14]}], "end": ["b"]},
    ]
    monkeypatch.setattr("sys.stdin", io.StringIO("".join(json.dumps(s) + "\n" for s in steps)))
    out = tmp_path / "out"
    out.mkdir()
    assert trace_run.main(["--model", str(checkpoint), "--dtype", dtype, "--out",
                           str(out), "--max-tokens", "128", "--device", device]) == 0
    assert capsys.readouterr().out.split("\n")[:4] == [f"done {k}" for k in (0, 1, 2, 7)]
    assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "7.f32"]
    ea, eb = cases.expected(NAME, a), cases.expected(NAME, b)
    for k, want in ((0, ea[[18, 0]]), (2, torch.stack([ea[23], eb[3], eb[4]])), (7, eb[19:])):
        got = torch.from_numpy(np.fromfile(out / f"{k}.f32", dtype="<f4").reshape(-1, 131))
        assert cases.model_error(got, want, getattr(torch, dtype)) < 1
