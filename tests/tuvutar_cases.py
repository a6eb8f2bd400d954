"""Small random Tuvutar models for the tests, and ways to run and compare."""

from __future__ import annotations

import json

import torch
from safetensors.torch import save_file

import tuvutar_oracle as oracle

YARN = {"factor": 4.0, "original": 256, "fast": 24.0, "slow": 1.0}


def delta(heads, kv_heads, dim, vdim, conv, ff=None):
    return {"type": "delta",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                      "vdim": vdim, "conv": conv},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def latent(heads, dim, rot, vdim, rank, ff=None, base=10000.0, scaling=None,
           scale=None, kv_from=None):
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim,
             "kv_rank": rank, "scale": scale or (dim + rot) ** -0.5,
             "rot": {"base": base, "dims": rot}}
    if scaling:
        mixer["rot"]["scaling"] = scaling
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": mixer,
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(width, vocab, layers, eps=1e-5):
    return {"architecture": "Tuvutar", "width": width, "vocab": vocab,
            "norm": {"eps": eps}, "layers": layers}


CONFIGS = {
    # unequal everything: grouped heads, odd sizes, both mlp cases, a shared
    # layer with other heads than its source, two rotations
    "mixed": config(96, 131, [
        delta(6, 2, 20, 36, 3),
        latent(3, 24, 16, 40, 48, ff=72, scaling=YARN),
        delta(2, 2, 16, 24, 5, ff=50),
        latent(5, 40, 16, 24, 48, scaling=YARN, kv_from=1, scale=0.21),
        latent(2, 32, 8, 16, 80, ff=64, base=500.0),
        delta(4, 4, 33, 17, 2, ff=40),
    ]),
    # ones: one head, one tap, one layer of each
    "ones": config(40, 67, [
        latent(1, 8, 2, 8, 8),
        delta(1, 1, 8, 8, 1, ff=24),
        latent(1, 16, 2, 4, 8, kv_from=0, ff=8),
    ], eps=1e-6),
    # attention first and last, no recurrence, factor 1
    "attention": config(64, 90, [
        latent(4, 16, 8, 16, 32, ff=96,
               scaling={"factor": 1.0, "original": 64, "fast": 8.0, "slow": 1.0}),
        latent(4, 16, 8, 16, 32, kv_from=0),
        latent(2, 48, 32, 72, 130, ff=33),
    ]),
    "recurrent": config(56, 71, [
        delta(3, 1, 48, 8, 8), delta(8, 4, 8, 64, 4, ff=48),
    ]),
}


def weights(cfg, seed=0):
    """Checkpoint tensors, bf16.  Decays reach from almost 1 to almost 0."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    out = {}

    def mat(name, rows, cols, gain=1.0):
        out[name] = torch.randn(rows, cols, generator=g) * gain * cols ** -0.5

    def vec(name, n, mean=0.0, std=0.2):
        out[name] = mean + std * torch.randn(n, generator=g)

    out["embed"] = torch.randn(cfg["vocab"], W, generator=g)
    for i, layer in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", layer["mixer"]
        m = p + "mix."
        vec(p + "norm1", W), vec(p + "norm1b", W)
        H, V = mx["heads"], mx["vdim"]
        if layer["type"] == "delta":
            for name, rows in (("q", mx["kv_heads"] * mx["dim"]),
                               ("k", mx["kv_heads"] * mx["dim"]), ("v", H * V)):
                mat(m + name, rows, W)
                mat(m + name + ".conv", rows, mx["conv"], 1.5)
            mat(m + "b", H, W), mat(m + "a", H, W), mat(m + "g", H * V, W)
            out[m + "A_log"] = torch.linspace(-5.0, 1.5, H) if H > 1 else \
                torch.tensor([-2.0])
            vec(m + "dt_bias", H, -1.0, 1.0)
            vec(m + "norm", V, 1.0)
        else:
            mat(m + "q", H * (mx["dim"] + mx["rot_dim"]), W, 1.6)
            if mx.get("kv_from") is None:
                mat(m + "dkv", mx["kv_rank"] + mx["rot_dim"], W, 1.6)
                vec(m + "dkv.norm", mx["kv_rank"], 1.0)
            mat(m + "uk", H * mx["dim"], mx["kv_rank"], 1.6)
            mat(m + "uv", H * V, mx["kv_rank"])
        mat(m + "o", W, H * V)
        if layer["mlp"] is not None:
            vec(p + "norm2", W), vec(p + "norm2b", W)
            ff = layer["mlp"]["ff"]
            mat(p + "mlp.gate", ff, W), mat(p + "mlp.up", ff, W)
            mat(p + "mlp.down", W, ff)
    vec("final.norm", W)
    mat("head", cfg["vocab"], W)
    return {k: v.to(torch.bfloat16).contiguous() for k, v in out.items()}


def write(path, cfg, w):
    path.mkdir(parents=True, exist_ok=True)
    save_file(w, str(path / "model.safetensors"))
    (path / "config.json").write_text(json.dumps(cfg))
    return path


def build(cfg, w, device="cpu", dtype=torch.float32, start=None, end=None):
    """The framework's stage model with these weights."""
    from mlx_sharding_amd.config import ModelConfig
    from mlx_sharding_amd.models import get_model_class
    from mlx_sharding_amd.models.fuse import fuse_model
    mc = ModelConfig.from_dict(json.loads(json.dumps(cfg)))
    cls = get_model_class(mc.model_type)
    cls.complete_config(mc, w)
    m = cls(mc, mc.shard(start, end))
    m.to(dtype)
    m.load_weights(w)
    m.to(device).eval()
    fuse_model(m)
    return m


def tokens(cfg, n, seed=1):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


_MEMO = {}


def expected(name, toks, seed=0):
    """Oracle logits of a named config, remembered."""
    key = (name, tuple(toks), seed)
    if key not in _MEMO:
        _MEMO[key] = oracle.forward(CONFIGS[name], weights(CONFIGS[name], seed), toks)
    return _MEMO[key]


def row_errors(got, want):
    """rms of the difference per row, over the rms of all rows."""
    got, want = got.double().cpu(), want.double().cpu()
    d = (got - want).pow(2).mean(-1).sqrt()
    assert torch.isfinite(d).all()
    return d / want.pow(2).mean().sqrt()


def error(got, want):
    return float(row_errors(got, want).max())


def model_error(got, want, dtype):
    """Error of a whole model in units of what is allowed.  In bf16 single
    rows may be off by more: a norm lifts small sublayer outputs together
    with their rounding."""
    e = row_errors(got, want)
    if dtype == torch.float32:
        return float(e.max()) / 5e-5
    return max(float(e.median()) / 4e-2, float(e.quantile(0.95)) / 0.15,
               float(e.max()) / 0.6)


def poison(state):
    """Make every use of storage that was never written show."""
    for layer in state.layers:
        if layer is not None:
            for t in (layer.rows, layer.state, layer.conv):
                if t is not None:
                    t.fill_(float("nan"))


def cut(n, sizes):
    """Portions of n tokens with these sizes, the last one repeated."""
    out, at, i = [], 0, 0
    while at < n:
        s = min(sizes[min(i, len(sizes) - 1)], n - at)
        out.append(s)
        at += s
        i += 1
    return out


def replay(engine, streams, schedule):
    """Run a schedule [[(id, n), ...], ...]; every token's logits per id.
    A request ends when its tokens are used up."""
    from mlx_sharding_amd.parallel.batching import Portion
    at = {r: 0 for r in streams}
    got = {r: [] for r in streams}
    for step in schedule:
        ps = [Portion(r, streams[r][at[r]: at[r] + n], range(n)) for r, n in step]
        logits = engine.step(ps).cpu()
        off = 0
        for r, n in step:
            got[r].append(logits[off: off + n])
            off += n
            at[r] += n
            if at[r] == len(streams[r]):
                engine.end(r)
    return {r: torch.cat(v) if v else None for r, v in got.items()}
