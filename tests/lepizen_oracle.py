"""Plain, slow oracle of the Lepizen design.

One function per mechanism, written from the equations: no cache, no batch, no
kernels, and nothing shared with the package under test.  A sequence is always
processed whole, in float64 unless told otherwise.
"""

from __future__ import annotations

import math

import torch


def rms_norm(x, w, eps):
    """Over the whole last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def gelu(z):
    """The exact one: z times the normal distribution function."""
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def softmax_with_sink(s, sink):
    """Rows of scores; the denominator has one term more, exp(sink)."""
    m = max(float(s.max()), float(sink))
    p = torch.exp(s - m)
    return p / (p.sum(-1, keepdim=True) + torch.exp(sink - m))


def mixed_values(v, first, lam):
    return (1.0 - lam) * v + lam * first


def attend(q, k, v, sink, scale):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim], sink [H]; head h reads
    key/value head h // (H / G); token i sees tokens 0..i."""
    T, H = q.shape[:2]
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        for i in range(T):
            s = (k[: i + 1, g] @ q[i, h]) * scale
            out[i, h] = softmax_with_sink(s, sink[h]) @ v[: i + 1, g]
    return out


def attend_rows(q, k, v, sink, scale):
    """The same, all tokens of a head at once."""
    T, H = q.shape[:2]
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    later = torch.ones(T, T).triu(1) > 0        # [query, key]
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].T) * scale).masked_fill(later, -math.inf)
        m = torch.maximum(s.max(-1, keepdim=True).values, sink[h])
        p = torch.exp(s - m)
        p = p / (p.sum(-1, keepdim=True) + torch.exp(sink[h] - m))
        out[:, h] = p @ v[:, g]
    return out


def attention(h, w, pre, mx, eps, first):
    """Returns (output, values before mixing).  first: the values that this
    layer mixes in, or None."""
    T = h.shape[0]
    H, G = mx["heads"], mx["kv_heads"]
    q = rms_norm(h @ w[pre + "q"].T, w[pre + "q.norm"], eps)
    k = rms_norm(h @ w[pre + "k"].T, w[pre + "k.norm"], eps)
    raw = v = h @ w[pre + "v"].T
    if first is not None:
        v = mixed_values(v, first, w[pre + "vmix"])
    o = attend_rows(q.reshape(T, H, mx["dim"]), k.reshape(T, G, mx["dim"]),
                    v.reshape(T, G, mx["vdim"]), w[pre + "sink"], mx["scale"])
    return o.reshape(T, -1) @ w[pre + "o"].T, raw


def mlp(h, w, pre):
    return gelu(h @ w[pre + "up"].T) @ w[pre + "down"].T


def cap(z, scale, limit):
    return limit * torch.tanh(z * scale / limit)


def forward(config, weights, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one whole sequence."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps, m = config["norm"]["eps"], config["residual_mult"]
    x = w["embed"][torch.as_tensor(tokens)]
    first = None
    for i, layer in enumerate(config["layers"]):
        p, mx = f"l{i}.", layer["mixer"]
        h = rms_norm(x, w[p + "norm1"], eps)
        y, raw = attention(h, w, p + "mix.", mx, eps,
                           first if mx["v_mix"] else None)
        if mx["v_mix"] and first is None:
            first = raw
        if layer["mlp"] is not None:
            y = y + mlp(h, w, p + "mlp.")
        x = x + m * y
        if layers_out is not None:
            layers_out.append(x.clone())
    z = rms_norm(x, w["final.norm"], eps) @ w["head"].T
    return cap(z, config["logit_scale"], config["logit_softcap"])
