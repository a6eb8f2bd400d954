"""Small random Dufinex models for the tests."""

from __future__ import annotations

import torch

import dufinex_oracle as oracle
from tuvutar_cases import build, cut, error, replay, row_errors, tokens, write  # noqa: F401


def dense(ff, limit=2.0):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(ff, experts, top, limit=2.0):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit},
            "router": {"experts": experts, "top": top}}


def attention(heads, kv_heads, dim, vdim, scale=None, kv_from=None, mlp=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
             "scale": scale or 2.0 * dim ** -0.5}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "attention", "mlp": mlp, "mixer": mixer}


def delta(heads, kv_heads, dim, vdim, conv, ranks=(6, 10), mlp=None):
    """ranks: of decay and gate; they stand in the tensors only."""
    return {"type": "channel_delta", "mlp": mlp, "ranks": ranks,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                      "vdim": vdim, "conv": conv}}


def config(width, vocab, layers, eps=1e-5, scale=1.5):
    return {"architecture": "Dufinex", "width": width, "vocab": vocab,
            "norm": {"eps": eps}, "embedding": {"scale": scale},
            "layers": layers}


CONFIGS = {
    # unequal everything: grouped heads in both mixers, sizes, ranks, both
    # feed-forwards and none, a source with two readers
    "mixed": config(96, 131, [
        attention(6, 2, 24, 40, mlp=moe(40, 5, 3)),
        delta(6, 2, 20, 36, 3, (12, 7), mlp=dense(50)),
        attention(6, 2, 24, 40, 0.7, kv_from=0),
        delta(4, 4, 33, 17, 2, (5, 9), mlp=moe(33, 7, 2, 0.8)),
        attention(6, 2, 24, 40, kv_from=0, mlp=dense(72, 0.5)),
        attention(4, 4, 40, 12, mlp=moe(24, 6, 1)),
    ]),
    # ones: one head, tap, channel, rank, unit, expert
    "ones": config(40, 67, [
        attention(1, 1, 2, 2, mlp=moe(1, 1, 1)),
        delta(1, 1, 8, 8, 1, (1, 1), mlp=dense(1)),
        attention(1, 1, 2, 2, kv_from=0, mlp=moe(4, 2, 1)),
    ], eps=1e-3, scale=1.0),
    # recurrent first and last, odd widths, eight taps, every expert chosen
    "odd": config(51, 71, [
        delta(3, 1, 19, 23, 8, (3, 5), mlp=moe(19, 4, 4)),
        attention(3, 3, 18, 7, mlp=dense(35)),
        delta(2, 1, 7, 5, 5, (9, 2)),
    ], scale=0.7),
    # may be cut into stages, but not between a source and its reader
    "stages": config(96, 131, [
        delta(6, 2, 20, 36, 3, (12, 7), mlp=dense(50)),
        attention(4, 2, 24, 16, mlp=dense(72, 1.2)),
        attention(4, 2, 24, 16, kv_from=1, mlp=moe(40, 5, 2)),
        delta(2, 2, 16, 24, 4, mlp=moe(33, 6, 1)),
        attention(3, 1, 16, 24),
    ]),
    # heads that the prompt kernels do not have, beside ones they do
    "wide": config(64, 90, [
        attention(4, 2, 72, 272, mlp=moe(72, 9, 2)),
        delta(2, 1, 160, 96, 4, (24, 16)),
        attention(4, 2, 72, 272, kv_from=0),
        delta(1, 1, 64, 200, 4, (8, 40), mlp=dense(130, 5.0)),
        attention(16, 2, 64, 256),
    ]),
}


def weights(cfg, seed=0):
    """Checkpoint tensors, bf16.  Decays reach from almost 1 to almost 0, within
    a head too, and many units meet their limits."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    out = {}

    def mat(name, rows, cols, gain=1.0):
        out[name] = torch.randn(rows, cols, generator=g) * gain * cols ** -0.5

    def vec(name, size, mean=0.0, std=0.2):
        out[name] = mean + std * torch.randn(size, generator=g)

    out["embed"] = torch.randn(cfg["vocab"], W, generator=g)
    for i, layer in enumerate(cfg["layers"]):
        p, mx, mlp = f"l{i}.", layer["mixer"], layer["mlp"]
        m = p + "mix."
        H, G, D, V = (mx[k] for k in ("heads", "kv_heads", "dim", "vdim"))
        vec(p + "norm1", W, 1.0)
        if layer["type"] == "attention":
            mat(m + "q", H * D, W), vec(m + "q.norm", D, 1.0)
            if mx.get("kv_from") is None:
                mat(m + "k", G * D, W), vec(m + "k.norm", D, 1.0)
                mat(m + "v", G * V, W)
            vec(m + "sink", H, 1.0, 1.0), mat(m + "g", H, W)
        else:
            ra, rg = layer["ranks"]
            for name, rows in (("q", G * D), ("k", G * D), ("v", H * V)):
                mat(m + name, rows, W), mat(m + name + ".conv", rows, mx["conv"], 1.5)
            mat(m + "b", H, W)
            mat(m + "a1", ra, W), mat(m + "a2", H * D, ra)
            mat(m + "g1", rg, W), mat(m + "g2", H * V, rg)
            out[m + "A_log"] = torch.linspace(-3.0, 1.0, H) if H > 1 else \
                torch.tensor([-1.5])
            vec(m + "dt_bias", H * D, -1.5, 2.0)
            vec(m + "norm", V, 1.0)
        mat(m + "o", W, H * V)
        if mlp is None:
            continue
        vec(p + "norm2", W, 1.0)
        if mlp["kind"] == "dense":
            for name, rows, cols in (("gate", mlp["ff"], W), ("up", mlp["ff"], W),
                                     ("down", W, mlp["ff"])):
                mat(f"{p}mlp.{name}", rows, cols), vec(f"{p}mlp.{name}.b", rows)
        else:
            ff = mlp["expert"]["ff"]
            mat(p + "mlp.router", mlp["router"]["experts"], W)
            for e in range(mlp["router"]["experts"]):
                mat(f"{p}mlp.e{e}.gate", ff, W, 2.0), mat(f"{p}mlp.e{e}.up", ff, W, 2.0)
                mat(f"{p}mlp.e{e}.down", W, ff)
    vec("final.norm", W, 1.0)
    return {k: v.to(torch.bfloat16).contiguous() for k, v in out.items()}


_MEMO = {}


def expected(name, toks, seed=0):
    """Oracle logits of a named config, remembered; a shorter sequence is the
    beginning of a longer one."""
    key = (name, seed)
    for known, logits in _MEMO.get(key, []):
        if list(known[: len(toks)]) == list(toks):
            return logits[: len(toks)]
    got = oracle.forward(CONFIGS[name], weights(CONFIGS[name], seed), toks)
    _MEMO.setdefault(key, []).append((tuple(toks), got))
    return got


def model_error(got, want, dtype):
    """Error of a whole model in units of what is allowed.  In bf16 a token's
    rounded router input may choose another expert, so single rows may be off."""
    e = row_errors(got, want)
    if dtype == torch.float32:
        return float(e.max()) / 1e-4
    return max(float(e.median()) / 6e-2, float(e.quantile(0.8)) / 0.4,
               float(e.max()) / 2.0)


def poison(state):
    """Make every use of storage that was never written show."""
    for layer in state.layers:
        for t in () if layer is None else (layer.rows, *layer.per_slot()):
            if t is not None:
                t.fill_(float("nan"))
