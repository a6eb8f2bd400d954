"""Small random Sadosun models for the tests."""

from __future__ import annotations

import torch

import sadosun_oracle as oracle
from tuvutar_cases import build, cut, error, replay, row_errors, tokens, write  # noqa: F401


def moe(ff, experts, top, identity=0):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top, "identity": identity}}


def attention(heads, kv_heads, dim, vdim, window, rot=None, base=10000.0,
              scale=None, mlp=None):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                      "vdim": vdim, "mask": {"size": window},
                      "rot": {"base": base, "dims": dim if rot is None else rot},
                      "scale": scale or 2.5 * dim ** -0.5}}


def mamba(inner, state, dt_rank, conv, mlp=None):
    return {"type": "mamba1", "mlp": mlp,
            "mixer": {"inner": inner, "state": state, "dt_rank": dt_rank,
                      "conv": conv}}


def config(width, vocab, layers, eps=1e-5, scale=3.0, taps=4, side=12):
    return {"architecture": "Sadosun", "width": width, "vocab": vocab,
            "norm": {"eps": eps}, "embedding": {"scale": scale},
            "canon": {"taps": taps}, "token_side": {"dim": side},
            "layers": layers}


CONFIGS = {
    # unequal everything: rotated part, key and value sizes, windows, bases,
    # states, taps, with and without experts and identity experts
    "mixed": config(96, 131, [
        attention(6, 2, 24, 40, 37, rot=16, mlp=moe(40, 5, 3, 2)),
        mamba(72, 12, 7, 3, mlp=moe(33, 6, 2)),
        attention(4, 4, 40, 12, 64, base=300.0),
        mamba(136, 40, 16, 5),
        attention(8, 1, 32, 32, 20, mlp=moe(64, 3, 1, 4)),
    ]),
    # ones: one head, tap, state, unit, expert; a window of one token
    "ones": config(40, 67, [
        attention(1, 1, 2, 2, 1, mlp=moe(1, 1, 1)),
        mamba(8, 1, 1, 1, mlp=moe(4, 1, 2, 1)),
        attention(2, 1, 8, 4, 1000),
    ], eps=1e-3, scale=1.0, taps=1, side=1),
    # the first layer recurrent, odd widths, two taps, every expert chosen
    "odd": config(51, 71, [
        mamba(37, 17, 5, 2, mlp=moe(19, 4, 6, 2)),
        attention(3, 3, 18, 6, 9, rot=2),
        mamba(64, 70, 3, 8, mlp=moe(8, 20, 8, 12)),
    ], taps=8, side=5),
    # heads that the prompt kernel does not have, beside ones it does
    "wide": config(64, 90, [
        attention(4, 2, 72, 272, 50, mlp=moe(72, 9, 2)),
        attention(2, 2, 272, 64, 70),
        attention(16, 2, 64, 256, 130),
    ], taps=2, side=64),
}


def weights(cfg, seed=0):
    """Checkpoint tensors, bf16.  Decays reach from almost 1 to almost 0, and
    the corrections change many choices."""
    g = torch.Generator().manual_seed(seed)
    W, n = cfg["width"], cfg["token_side"]["dim"]
    out = {}

    def mat(name, rows, cols, gain=1.0):
        out[name] = torch.randn(rows, cols, generator=g) * gain * cols ** -0.5

    def vec(name, size, mean=0.0, std=0.2):
        out[name] = mean + std * torch.randn(size, generator=g)

    out["embed"] = torch.randn(cfg["vocab"], W, generator=g)
    out["side.embed"] = torch.randn(cfg["vocab"], n * len(cfg["layers"]), generator=g)
    for i, lay in enumerate(cfg["layers"]):
        p, mx, mlp = f"l{i}.", lay["mixer"], lay["mlp"]
        m = p + "mix."
        vec(p + "norm1", (), 1.1)
        mat(p + "canon1", W, cfg["canon"]["taps"])
        if lay["type"] == "attention":
            H, G, D, V = (mx[k] for k in ("heads", "kv_heads", "dim", "vdim"))
            mat(m + "q", H * D, W), mat(m + "k", G * D, W)
            mat(m + "v", G * V, W, 1.5), mat(m + "o", W, H * V, 2.0)
        else:
            C, N, R = mx["inner"], mx["state"], mx["dt_rank"]
            mat(m + "in", 2 * C, W, 1.5)
            mat(m + "conv", C, mx["conv"], 1.2), vec(m + "conv.b", C)
            mat(m + "x", R + 2 * N, C, 1.5)
            mat(m + "dt", C, R), vec(m + "dt.b", C, -1.5, 1.5)
            out[m + "A_log"] = torch.linspace(-3.0, 2.0, N).expand(C, N) \
                + 0.3 * torch.randn(C, N, generator=g)
            vec(m + "D", C, 0.5), mat(m + "o", W, C, 2.0)
        if mlp is not None:
            r, ff = mlp["router"], mlp["expert"]["ff"]
            total = r["experts"] + r["identity"]
            vec(p + "norm2", (), 0.9)
            mat(p + "canon2", W, cfg["canon"]["taps"])
            mat(p + "mlp.router", total, W, 2.0)
            vec(p + "mlp.correction", total, 0.1)
            for e in range(r["experts"]):
                mat(f"{p}mlp.e{e}.up", ff, W), mat(f"{p}mlp.e{e}.down", W, ff)
        mat(p + "side.gate", n, W), mat(p + "side.proj", W, n)
        vec(p + "side.norm", W, 0.7)
    vec("final.norm", (), 1.2)
    mat("head", cfg["vocab"], W, 2.0)
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
    return max(float(e.median()) / 6e-2, float(e.quantile(0.9)) / 0.4,
               float(e.max()) / 2.0)


def poison(state):
    """Make every use of storage that was never written show."""
    for layer in state.layers:
        for t in (layer.rows, *layer.per_slot()):
            if t is not None:
                t.fill_(float("nan"))
