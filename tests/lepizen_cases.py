"""Small random Lepizen models for the tests."""

from __future__ import annotations

import torch

import lepizen_oracle as oracle
from tuvutar_cases import (build, cut, error, poison, replay, row_errors,  # noqa: F401
                           tokens, write)


def layer(heads, kv_heads, dim, vdim, scale=None, v_mix=True, ff=None):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                      "vdim": vdim, "scale": scale or dim ** -0.5,
                      "v_mix": v_mix},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(width, vocab, layers, eps=1e-5, mult=0.6, scale=0.7, cap=8.0):
    return {"architecture": "Lepizen", "width": width, "vocab": vocab,
            "norm": {"eps": eps}, "residual_mult": mult, "logit_scale": scale,
            "logit_softcap": cap, "layers": layers}


CONFIGS = {
    # unequal everything: the first mixing layer in the middle, one without
    # mixing behind it, kinds of grouping, both mlp cases, odd sizes
    "mixed": config(96, 131, [
        layer(6, 2, 24, 40, ff=72, v_mix=False),
        layer(4, 4, 40, 12, scale=0.3),
        layer(9, 3, 17, 21, ff=50, v_mix=False),
        layer(8, 2, 32, 24, scale=0.11, ff=97),
        layer(12, 1, 48, 48, ff=64),
    ]),
    # ones: one head, one feed-forward unit, constants of 1
    "ones": config(40, 67, [
        layer(1, 1, 8, 8, scale=1.0, ff=1),
        layer(1, 1, 16, 8),
    ], eps=1e-6, mult=1.0, scale=1.0, cap=1.0),
    # nothing mixes
    "plain": config(56, 71, [
        layer(4, 2, 16, 16, v_mix=False, ff=48),
        layer(2, 2, 64, 32, v_mix=False),
    ], mult=0.25, cap=30.0),
    # heads that the prompt kernel does not have, beside ones it does
    "wide": config(64, 90, [
        layer(4, 2, 72, 272, ff=40),
        layer(2, 2, 272, 272),
        layer(4, 2, 264, 272, ff=32),
        layer(16, 2, 64, 272),
    ]),
}


def weights(cfg, seed=0):
    """Checkpoint tensors, bf16.  Sinks are of the order of the scores."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    out = {}

    def mat(name, rows, cols, gain=1.0):
        out[name] = torch.randn(rows, cols, generator=g) * gain * cols ** -0.5

    def vec(name, n, mean=1.0, std=0.2):
        out[name] = mean + std * torch.randn(n, generator=g)

    out["embed"] = torch.randn(cfg["vocab"], W, generator=g)
    for i, lay in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", lay["mixer"]
        m = p + "mix."
        H, G, D, V = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
        vec(p + "norm1", W)
        mat(m + "q", H * D, W), mat(m + "k", G * D, W), mat(m + "v", G * V, W)
        vec(m + "q.norm", H * D, 1.3), vec(m + "k.norm", G * D, 1.3)
        out[m + "sink"] = 3.0 + 1.5 * torch.randn(H, generator=g)
        if mx["v_mix"]:
            out[m + "vmix"] = torch.rand((), generator=g)
        mat(m + "o", W, H * V, 2.0)
        if lay["mlp"] is not None:
            ff = lay["mlp"]["ff"]
            mat(p + "mlp.up", ff, W, 1.5), mat(p + "mlp.down", W, ff)
    vec("final.norm", W)
    mat("head", cfg["vocab"], W, 4.0)
    return {k: v.to(torch.bfloat16).contiguous() for k, v in out.items()}


_MEMO = {}


def expected(name, toks, seed=0):
    """Oracle logits of a named config, remembered."""
    key = (name, tuple(toks), seed)
    if key not in _MEMO:
        _MEMO[key] = oracle.forward(CONFIGS[name], weights(CONFIGS[name], seed), toks)
    return _MEMO[key]


def model_error(got, want, dtype):
    """Error of a whole model in units of what is allowed."""
    return error(got, want) / (2e-5 if dtype == torch.float32 else 4e-2)
