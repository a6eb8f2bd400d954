"""Plain, slow oracle of the Tuvutar design.

One function per mechanism, written from the equations: no cache, no batch, no
chunks, no kernels, and nothing shared with the package under test.  A sequence
is always processed whole, token after token or key after key, in float64
unless told otherwise.
"""

from __future__ import annotations

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_around_zero(x, w, eps):
    return rms(x, eps) * (1.0 + w)


def norm_plain(x, w, eps):
    return rms(x, eps) * w


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def silu(x):
    return x / (1.0 + torch.exp(-x))


def gelu_tanh(x):
    return 0.5 * x * (1.0 + torch.tanh(
        math.sqrt(2.0 / math.pi) * (x + 0.044715 * x ** 3)))


def softplus(x):
    return torch.clamp(x, min=0) + torch.log1p(torch.exp(-x.abs()))


def rotary_frequencies(rot):
    """(frequency per pair, factor on cos and sin)."""
    dims, base = rot["dims"], rot["base"]
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def dim_of(turns):
        return (dims * math.log(sc["original"] / (2 * math.pi * turns))
                / (2 * math.log(base)))

    lo = max(math.floor(dim_of(sc["fast"])), 0)
    hi = min(math.ceil(dim_of(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * ramp + fi * (1.0 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, rot):
    """x [T, ..., dims]; pairs are neighbours; the row index is the position."""
    f, m = rotary_frequencies(rot)
    f = torch.tensor(f, dtype=torch.float64)
    y = torch.empty_like(x)
    for p in range(x.shape[0]):
        c, s = (torch.cos(p * f) * m).to(x.dtype), (torch.sin(p * f) * m).to(x.dtype)
        u, v = x[p, ..., 0::2], x[p, ..., 1::2]
        y[p, ..., 0::2] = u * c - v * s
        y[p, ..., 1::2] = v * c + u * s
    return y


def latent_rows(h, w, pre, mx, eps):
    """The two things a latent layer caches: normed latent, rotated key part."""
    r = mx["kv_rank"]
    d = h @ w[pre + "dkv"].T
    c = norm_plain(d[:, :r], w[pre + "dkv.norm"], eps)
    return c, rotate(d[:, r:], mx["rot"])


def latent_attention(h, w, pre, mx, c, kr):
    T = h.shape[0]
    H, dim, rd, vd = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"]
    q = (h @ w[pre + "q"].T).reshape(T, H, dim + rd)
    qn, qr = q[..., :dim], rotate(q[..., dim:], mx["rot"])
    k = (c @ w[pre + "uk"].T).reshape(T, H, dim)
    v = (c @ w[pre + "uv"].T).reshape(T, H, vd)
    out = torch.zeros(T, H, vd, dtype=h.dtype)
    seen = torch.ones(T, T).tril() > 0      # [query, key]
    for a in range(H):
        s = (qn[:, a] @ k[:, a].T + qr[:, a] @ kr.T) * mx["scale"]
        s = torch.where(seen, s, torch.full_like(s, -math.inf))
        p = torch.exp(s - s.max(-1, keepdim=True).values)
        out[:, a] = (p / p.sum(-1, keepdim=True)) @ v[:, a]
    return out.reshape(T, H * vd) @ w[pre + "o"].T


def short_conv(x, taps):
    """x [T, C], taps [C, K], the last column meets the current token."""
    T, K = x.shape[0], taps.shape[1]
    y = torch.zeros_like(x)
    for back in range(min(K, T)):           # how many tokens ago
        y[back:] += taps[:, K - 1 - back] * x[: T - back]
    return y


def delta_rule(q, k, v, beta, g):
    """q, k [T, H, D] (q and k ready), v [T, H, V], beta, g [T, H]."""
    T, H, D = q.shape
    V = v.shape[-1]
    o = torch.zeros(T, H, V, dtype=q.dtype)
    S = torch.zeros(H, D, V, dtype=q.dtype)
    for t in range(T):
        S = g[t, :, None, None] * S
        u = beta[t, :, None] * (v[t] - (S * k[t, :, :, None]).sum(1))
        S = S + k[t, :, :, None] * u[:, None, :]
        o[t] = (S * q[t, :, :, None]).sum(1)
    return o


def delta(h, w, pre, mx, eps):
    T = h.shape[0]
    H, KH, D, V = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]

    def lane(name, heads, size):
        x = silu(short_conv(h @ w[pre + name].T, w[pre + name + ".conv"]))
        return x.reshape(T, heads, size)

    q = unit(lane("q", KH, D)) * D ** -0.5
    k = unit(lane("k", KH, D))
    v = lane("v", H, V)
    idx = [a // (H // KH) for a in range(H)]
    beta = 1.0 / (1.0 + torch.exp(-(h @ w[pre + "b"].T)))
    g = torch.exp(-torch.exp(w[pre + "A_log"])
                  * softplus(h @ w[pre + "a"].T + w[pre + "dt_bias"]))
    o = delta_rule(q[:, idx], k[:, idx], v, beta, g)
    gate = silu(h @ w[pre + "g"].T).reshape(T, H, V)
    o = rms(o, eps) * w[pre + "norm"] * gate
    return o.reshape(T, H * V) @ w[pre + "o"].T


def dense_mlp(h, w, pre):
    return (gelu_tanh(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def forward(config, weights, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one whole sequence."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)]
    cached = {}
    for i, layer in enumerate(config["layers"]):
        p, mx = f"l{i}.", layer["mixer"]
        h = norm_around_zero(x, w[p + "norm1"], eps)
        if layer["type"] == "delta":
            y = delta(h, w, p + "mix.", mx, eps)
        else:
            src = mx.get("kv_from")
            if src is None:
                cached[i] = latent_rows(h, w, p + "mix.", mx, eps)
                src = i
            y = latent_attention(h, w, p + "mix.", mx, *cached[src])
        x = x + norm_around_zero(y, w[p + "norm1b"], eps)
        if layer["mlp"] is not None:
            h = norm_around_zero(x, w[p + "norm2"], eps)
            x = x + norm_around_zero(dense_mlp(h, w, p + "mlp."), w[p + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return norm_around_zero(x, w["final.norm"], eps) @ w["head"].T
