"""Plain, slow oracle of the Sadosun design.

One function per mechanism, written from the equations: no cache, no batch, no
kernels, and nothing shared with the package under test.  A sequence is always
processed whole, in float64 unless told otherwise.
"""

from __future__ import annotations

import math

import torch


# -- pieces -----------------------------------------------------------------

def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi)
                                       * (z + 0.044715 * z ** 3)))


def silu(z):
    return z / (1.0 + torch.exp(-z))


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def causal_conv(h, w):
    """h [T, C], w [C, taps]; the last tap meets the current row."""
    T, taps = h.shape[0], w.shape[1]
    out = torch.zeros_like(h)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                out[t] += w[:, j] * h[s]
    return out


def with_recent(h, w):
    """What a sublayer reads: its rows plus a convolution of them."""
    return h + causal_conv(h, w)


def turn(x, pos, base, dims, sign=1.0):
    """Rotate neighbouring pairs of the first ``dims`` of the last axis.
    x [T, heads, size], pos [T]."""
    out = x.clone()
    for i in range(dims // 2):
        a = sign * pos.to(torch.float64) * float(base) ** (-2.0 * i / dims)
        c, s = (f(a).to(x.dtype)[:, None] for f in (torch.cos, torch.sin))
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


# -- attention --------------------------------------------------------------

def attend(q, k, v, scale, window):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim]; head h reads key/value
    head h // (H / G); token i sees the last ``window`` tokens up to itself;
    one is added to every denominator."""
    T, H = q.shape[:2]
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        for i in range(T):
            lo = max(0, i - window + 1)
            e = torch.exp((k[lo: i + 1, g] @ q[i, h]) * scale)
            out[i, h] = (e / (1.0 + e.sum())) @ v[lo: i + 1, g]
    return out


def attend_rows(q, k, v, scale, window):
    """The same, all tokens of a head at once."""
    T, H = q.shape[:2]
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    i = torch.arange(T)
    gap = i[:, None] - i[None, :]
    hidden = (gap < 0) | (gap >= window)
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].T) * scale).masked_fill(hidden, -math.inf)
        m = s.max(-1, keepdim=True).values.clamp(min=0.0)
        p = torch.exp(s - m)
        out[:, h] = (p / (p.sum(-1, keepdim=True) + torch.exp(-m))) @ v[:, g]
    return out


def attention(h, w, pre, mx, eps):
    T = h.shape[0]
    H, G, D, V = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    pos = torch.arange(T)
    base, dims = mx["rot"]["base"], mx["rot"]["dims"]
    q = (h @ w[pre + "q"].T).reshape(T, H, D)
    k = (h @ w[pre + "k"].T).reshape(T, G, D)
    v = (h @ w[pre + "v"].T).reshape(T, G, V)
    q = rms(turn(q, pos, base, dims), eps)
    k = rms(turn(k, pos, base, dims), eps)
    v = turn(v, pos, base, V)
    o = attend_rows(q, k, v, mx["scale"], mx["mask"]["size"])
    o = turn(o, pos, base, V, -1.0)
    return o.reshape(T, H * V) @ w[pre + "o"].T


# -- selective scan ---------------------------------------------------------

def scan(x, dt, A, B, C, D):
    """x, dt [T, channels], A [channels, N], B, C [T, N], D [channels]."""
    S = torch.zeros_like(A)
    y = torch.zeros_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + D * x[t]
    return y


def mamba(h, w, pre, mx):
    R, N = mx["dt_rank"], mx["state"]
    x, z = (h @ w[pre + "in"].T).split([mx["inner"], mx["inner"]], 1)
    x = silu(causal_conv(x, w[pre + "conv"]) + w[pre + "conv.b"])
    dt, B, C = (x @ w[pre + "x"].T).split([R, N, N], 1)
    dt = softplus(dt @ w[pre + "dt"].T + w[pre + "dt.b"])
    y = scan(x, dt, -torch.exp(w[pre + "A_log"]), B, C, w[pre + "D"])
    return (y * silu(z)) @ w[pre + "o"].T


# -- experts ----------------------------------------------------------------

def route(z, correction, top):
    """Router logits [T, experts] -> (chosen [T, top], their weights)."""
    s = torch.softmax(z, -1)
    chosen = torch.topk(s + correction, top, dim=-1).indices
    picked = s.gather(-1, chosen)
    return chosen, picked / (picked.sum(-1, keepdim=True) + 1e-20)


def experts(h, w, pre, mlp):
    n, top = mlp["router"]["experts"], mlp["router"]["top"]
    chosen, weight = route(h @ w[pre + "router"].T, w[pre + "correction"], top)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, g in zip(chosen[t].tolist(), weight[t]):
            if e >= n:
                y = h[t]
            else:
                u = torch.clamp(w[f"{pre}e{e}.up"] @ h[t], min=0.0) ** 2
                y = w[f"{pre}e{e}.down"] @ u
            out[t] += g * y
    return out


# -- token input of a layer -------------------------------------------------

def token_input(x, e, w, pre, eps):
    g = gelu_tanh(x @ w[pre + "gate"].T) * e
    return rms(g @ w[pre + "proj"].T, eps) * w[pre + "norm"]


# -- model ------------------------------------------------------------------

def forward(config, weights, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one whole sequence."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps, n = config["norm"]["eps"], config["token_side"]["dim"]
    ids = torch.as_tensor(tokens)
    x = w["embed"][ids] * config["embedding"]["scale"]
    for i, layer in enumerate(config["layers"]):
        p, mx = f"l{i}.", layer["mixer"]
        h = with_recent(rms(x, eps) * w[p + "norm1"], w[p + "canon1"])
        if layer["type"] == "attention":
            x = x + attention(h, w, p + "mix.", mx, eps)
        else:
            x = x + mamba(h, w, p + "mix.", mx)
        if layer["mlp"] is not None:
            h = with_recent(rms(x, eps) * w[p + "norm2"], w[p + "canon2"])
            x = x + experts(h, w, p + "mlp.", layer["mlp"])
        x = x + token_input(x, w["side.embed"][ids][:, i * n: (i + 1) * n], w,
                            p + "side.", eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T
