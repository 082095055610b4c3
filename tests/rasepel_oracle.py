"""Plain, slow PyTorch rendering of the Rasepel decoder, one function per mechanism.

Everything runs with explicit loops over tokens (and heads, keys, blocks) in one precision
(float64 by default), straight from the equations; it shares nothing with the engine's model,
cache or kernels.  A model is a ``config`` dict (the keys of a Rasepel ``config.json``) and a
dict of tensors named as in its checkpoint.

Layer:  x <- x + N(mixer(x), norm1), then x <- x + N(ff(x), norm2), where
N(y, w) = y / sqrt(mean y^2 + eps) * (1 + w): the norm sits on what a sublayer produces only.
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.where(z > 0, z, torch.zeros_like(z)) + torch.log1p(torch.exp(-z.abs()))


def short_conv(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), nothing before token 0."""
    T, taps = u.shape[0], w.shape[1]
    y = torch.zeros_like(u)
    for s in range(T):
        for j in range(taps):
            i = s - taps + 1 + j
            if i >= 0:
                y[s] += w[:, j] * u[i]
    return y


# ------------------------------------------------------------------ lightning attention
def decayed_memory(q, k, v, decay):
    """q, k [T, H, D], v [T, H, V]: per head S <- decay_h S + k v^T, o = S^T q."""
    T, H, D = q.shape
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for hd in range(H):
        S = torch.zeros(D, v.shape[2], dtype=q.dtype)
        for s in range(T):
            S = decay[hd] * S + k[s, hd][:, None] * v[s, hd][None, :]
            out[s, hd] = S.T @ q[s, hd]
    return out


def lightning(h, t, p, mx, eps):
    H, D, V = mx["heads"], mx["dim"], mx["vdim"]
    T = h.shape[0]
    q, k, v = (silu(h @ t[p + n].T) for n in ("q", "k", "v"))
    o = decayed_memory(q.view(T, H, D), k.view(T, H, D), v.view(T, H, V), mx["decay"])
    o = rms(o.reshape(T, H * V), eps) * t[p + "norm"]        # one mean square over all heads
    return (o * torch.sigmoid(h @ t[p + "g"].T)) @ t[p + "o"].T


# ------------------------------------------------------------------ selective scan
def selective_scan(x, dt, A, B, C, D):
    """x, dt [T, I], A [I, N], B, C [T, N], D [I]."""
    S = torch.zeros_like(A)
    y = torch.zeros_like(x)
    for s in range(x.shape[0]):
        S = torch.exp(dt[s][:, None] * A) * S + (dt[s] * x[s])[:, None] * B[s][None, :]
        y[s] = S @ C[s] + D * x[s]
    return y


def mamba1(h, t, p, mx, eps):
    inner, N, rank = mx["inner"], mx["state"], mx["dt_rank"]
    xz = h @ t[p + "in"].T
    x = silu(short_conv(xz[:, :inner], t[p + "conv"]) + t[p + "conv.b"])
    xp = x @ t[p + "x"].T
    dt = softplus(xp[:, :rank] @ t[p + "dt"].T + t[p + "dt.b"])
    y = selective_scan(x, dt, -torch.exp(t[p + "A_log"]), xp[:, rank:rank + N], xp[:, rank + N:], t[p + "D"])
    return (y * silu(xz[:, inner:])) @ t[p + "o"].T


# ------------------------------------------------------------------ attention
def rotate_halves(x, dims, base):
    """x [T, heads, n]: channels (i, i + dims/2), i < dims/2, turned by position * base^(-2i/dims)."""
    out = x.clone()
    for s in range(x.shape[0]):
        for i in range(dims // 2):
            a = s * base ** (-2.0 * i / dims)
            c, sn = math.cos(a), math.sin(a)
            u, v = x[s, :, i], x[s, :, i + dims // 2]
            out[s, :, i] = u * c - v * sn
            out[s, :, i + dims // 2] = v * c + u * sn
    return out


def visible(position, size, pool):
    """(token positions, blocks) that a query at ``position`` sees: the last ``size`` tokens, and
    every block of ``pool`` tokens that ends at least ``size`` positions back."""
    tokens = [j for j in range(position + 1) if position - j < size]
    blocks = []
    b = 0
    while pool and b * pool + pool - 1 <= position - size:
        blocks.append(b)
        b += 1
    return tokens, blocks


def attention(h, t, p, mx, eps):
    H, G, D, V = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    size, P = mx["mask"]["size"], mx["mask"].get("pool")
    T = h.shape[0]
    q, k, v = (short_conv(h @ t[p + n].T + t[p + n + ".b"], t[p + n + ".conv"]) for n in ("q", "k", "v"))
    rot = mx.get("rot")
    q, k, v = q.view(T, H, D), k.view(T, G, D), v.view(T, G, V)
    if rot:
        q, k = (rotate_halves(z, rot["dims"], float(rot["base"])) for z in (q, k))
    q, k = rms(q, eps), rms(k, eps)
    gate = torch.sigmoid(h @ t[p + "g"].T)
    out = torch.zeros(T, H, V, dtype=h.dtype)
    for s in range(T):
        tokens, blocks = visible(s, size, P)
        ks = [k[j] for j in tokens] + [k[b * P:b * P + P].mean(0) for b in blocks]
        vs = [v[j] for j in tokens] + [v[b * P:b * P + P].mean(0) for b in blocks]
        ks, vs = torch.stack(ks), torch.stack(vs)                        # [n, G, .]
        for hd in range(H):
            g = hd // (H // G)
            w = torch.softmax((ks[:, g] @ q[s, hd]) * float(mx["scale"]) * t[p + "temp"][hd], 0)
            out[s, hd] = (w[:, None] * vs[:, g]).sum(0)
    return (out.reshape(T, H * V) * gate) @ t[p + "o"].T + t[p + "o.b"]


MIXERS = {"lightning": lightning, "mamba1": mamba1, "attention": attention}


# ------------------------------------------------------------------ feed-forward
def clamped_unit(h, t, p, limit):
    g = torch.clamp(h @ t[p + "gate"].T, max=limit)
    u = torch.clamp(h @ t[p + "up"].T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ t[p + "down"].T


# ------------------------------------------------------------------ model
def forward(config, t, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one sequence run from position 0."""
    t = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in t.items()}
    eps = float(config["norm"]["eps"])
    x = t["embed"][torch.tensor(tokens)] * float(config["embedding"]["scale"])
    for i, L in enumerate(config["layers"]):
        p = "l%d." % i
        x = x + rms(MIXERS[L["type"]](x, t, p + "mix.", L["mixer"], eps), eps) * (1 + t[p + "norm1"])
        if L.get("mlp"):
            y = clamped_unit(x, t, p + "mlp.", float(L["mlp"]["limit"]))
            x = x + rms(y, eps) * (1 + t[p + "norm2"])
        if layers_out is not None:
            layers_out.append(x.clone())
    return (rms(x, eps) * (1 + t["final.norm"])) @ t["embed"].T
