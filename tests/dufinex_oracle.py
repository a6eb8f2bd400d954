"""Plain, slow oracle of the Dufinex design.

One function per mechanism, written from the equations: no cache, no batch, no
chunks, no kernels, and nothing shared with the package under test.  A sequence
is always processed whole, in float64 unless told otherwise.
"""

from __future__ import annotations

import math

import torch


# -- pieces -----------------------------------------------------------------

def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def causal_conv(x, w):
    """x [T, C], w [C, taps]; the last tap meets the current row."""
    T, taps = x.shape[0], w.shape[1]
    y = torch.zeros_like(x)
    for back in range(min(taps, T)):
        y[back:] += w[:, taps - 1 - back] * x[: T - back]
    return y


def clamped_glu(g, u, limit):
    g, u = torch.clamp(g, max=limit), torch.clamp(u, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


# -- attention --------------------------------------------------------------

def attend(q, k, v, scale, sink):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim]; head h reads key/value head
    h // (H / G), and its denominator has exp(sink[h]) besides."""
    T, H = q.shape[:2]
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        for i in range(T):
            s = (k[: i + 1, g] @ q[i, h]) * scale
            m = torch.maximum(s.max(), sink[h])
            p = torch.exp(s - m)
            out[i, h] = (p @ v[: i + 1, g]) / (p.sum() + torch.exp(sink[h] - m))
    return out


def attend_rows(q, k, v, scale, sink):
    """The same, all tokens of a head at once."""
    T, H = q.shape[:2]
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    later = torch.ones(T, T).triu(1) > 0
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].T) * scale).masked_fill(later, -math.inf)
        m = torch.maximum(s.max(-1, keepdim=True).values, sink[h])
        p = torch.exp(s - m)
        out[:, h] = (p @ v[:, g]) / (p.sum(-1, keepdim=True) + torch.exp(sink[h] - m))
    return out


def keys_values(h, w, pre, mx, eps):
    """What a layer with its own projections keeps of each token."""
    T, G = h.shape[0], mx["kv_heads"]
    k = (h @ w[pre + "k"].T).reshape(T, G, mx["dim"])
    v = (h @ w[pre + "v"].T).reshape(T, G, mx["vdim"])
    return rms(k, eps) * w[pre + "k.norm"], v


def attention(h, w, pre, mx, eps, k, v):
    T, H = h.shape[0], mx["heads"]
    q = (h @ w[pre + "q"].T).reshape(T, H, mx["dim"])
    q = rms(q, eps) * w[pre + "q.norm"]
    o = attend_rows(q, k, v, mx["scale"], w[pre + "sink"])
    o = o * sigmoid(h @ w[pre + "g"].T)[:, :, None]
    return o.reshape(T, -1) @ w[pre + "o"].T


# -- delta rule with a decay per channel ------------------------------------

def delta_rule(q, k, v, beta, g):
    """q, k, g [T, H, D], v [T, H, V], beta [T, H]."""
    T, H, D = q.shape
    o = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype)
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    return o


def channel_delta(h, w, pre, mx, eps):
    T = h.shape[0]
    H, KH, D, V = (mx[n] for n in ("heads", "kv_heads", "dim", "vdim"))

    def lane(name, heads, size):
        x = silu(causal_conv(h @ w[pre + name].T, w[pre + name + ".conv"]))
        return x.reshape(T, heads, size)

    idx = [a // (H // KH) for a in range(H)]
    q = (unit(lane("q", KH, D)) * D ** -0.5)[:, idx]
    k = unit(lane("k", KH, D))[:, idx]
    v = lane("v", H, V)
    beta = sigmoid(h @ w[pre + "b"].T)
    a = (h @ w[pre + "a1"].T) @ w[pre + "a2"].T
    rate = torch.exp(w[pre + "A_log"])[:, None]
    g = torch.exp(-rate * softplus(a + w[pre + "dt_bias"]).reshape(T, H, D))
    o = rms(delta_rule(q, k, v, beta, g), eps) * w[pre + "norm"]
    gate = sigmoid((h @ w[pre + "g1"].T) @ w[pre + "g2"].T).reshape(T, H, V)
    return (o * gate).reshape(T, H * V) @ w[pre + "o"].T


# -- feed-forward -----------------------------------------------------------

def dense(h, w, pre, limit):
    g = h @ w[pre + "gate"].T + w[pre + "gate.b"]
    u = h @ w[pre + "up"].T + w[pre + "up.b"]
    return clamped_glu(g, u, limit) @ w[pre + "down"].T + w[pre + "down.b"]


def route(z, top):
    """Router logits [T, experts] -> (chosen [T, top], their weights)."""
    s = sigmoid(z)
    chosen = torch.topk(s, top, dim=-1).indices
    return chosen, s.gather(-1, chosen)


def experts(h, w, pre, mlp):
    limit = mlp["expert"]["limit"]
    chosen, weight = route(h @ w[pre + "router"].T, mlp["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(chosen[t].tolist(), weight[t]):
            x, p = s * h[t], f"{pre}e{e}."
            y = clamped_glu(w[p + "gate"] @ x, w[p + "up"] @ x, limit)
            out[t] += w[p + "down"] @ y
    return out


# -- model ------------------------------------------------------------------

def forward(config, weights, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one whole sequence."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)] * config["embedding"]["scale"]
    kept = {}
    for i, layer in enumerate(config["layers"]):
        p, mx, mlp = f"l{i}.", layer["mixer"], layer["mlp"]
        if layer["type"] == "attention":
            src = mx.get("kv_from")
            if src is None:
                src = i
                kept[i] = keys_values(x, w, p + "mix.", mx, eps)
            y = attention(x, w, p + "mix.", mx, eps, *kept[src])
        else:
            y = channel_delta(x, w, p + "mix.", mx, eps)
        x = x + rms(y, eps) * w[p + "norm1"]
        if mlp is not None:
            if mlp["kind"] == "dense":
                y = dense(x, w, p + "mlp.", mlp["limit"])
            else:
                y = experts(x, w, p + "mlp.", mlp)
            x = x + rms(y, eps) * w[p + "norm2"]
        if layers_out is not None:
            layers_out.append(x.clone())
    return (rms(x, eps) * w["final.norm"]) @ w["embed"].T
