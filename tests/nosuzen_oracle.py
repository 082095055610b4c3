"""Plain, slow PyTorch rendering of the Nosuzen decoder, one function per mechanism.

Everything runs with explicit loops over tokens, heads and keys in one precision (float64 by
default), straight from the equations; it shares nothing with the engine's model, cache or
kernels.  A model is a ``config`` dict (the keys of a Nosuzen ``config.json``) and a dict of
tensors named as in its checkpoint.

The residual is a bundle of streams X_1 .. X_n, all equal to the scaled embedding at first.  A
sublayer f with the coefficients a (in), M (mix) and c (out) reads u = sum_s a_s X_s and replaces
all streams at once, X_t <- sum_s M[s, t] X_s + c_t f(N(u)); N is tanh(alpha x) w + b.
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


# ------------------------------------------------------------------ norm and residual
def dynamic_tanh(x, t, name):
    return torch.tanh(t[name + ".alpha"] * x) * t[name] + t[name + ".b"]


def read_streams(X, coef):
    """X: list of streams -> sum_s coef[s] X_s."""
    u = torch.zeros_like(X[0])
    for s, x in enumerate(X):
        u = u + coef[s] * x
    return u


def write_streams(X, mix, out, y):
    new = []
    for to in range(len(X)):
        z = out[to] * y
        for frm in range(len(X)):
            z = z + mix[frm, to] * X[frm]
        new.append(z)
    return new


# ------------------------------------------------------------------ rotation
def rotation(rot):
    """(frequencies, factor on cos and sin) of a ``rot`` dict; ``scaling`` is YaRN's."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    factor, original = float(sc["factor"]), float(sc["original"])
    where = lambda turns: dims * math.log(original / (2 * math.pi * turns)) / (2 * math.log(base))
    lo = max(math.floor(where(float(sc["fast"]))), 0)
    hi = min(math.ceil(where(float(sc["slow"]))), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / factor * ramp + fi * (1 - ramp))
    return out, 0.1 * math.log(factor) + 1.0


def rotate(x, positions, rot, half):
    """x [T, ..., n]: the first rot.dims channels turned, pairs (i, i + dims/2) with ``half``, else
    (2i, 2i+1)."""
    f, m = rotation(rot)
    out = x.clone()
    for s, p in enumerate(positions):
        for i, fi in enumerate(f):
            a, b = (i, i + len(f)) if half else (2 * i, 2 * i + 1)
            c, sn = m * math.cos(p * fi), m * math.sin(p * fi)
            u, v = x[s, ..., a], x[s, ..., b]
            out[s, ..., a] = u * c - v * sn
            out[s, ..., b] = v * c + u * sn
    return out


# ------------------------------------------------------------------ visibility
def visible(i, mask):
    """Positions that position i sees: the window, and the kept first tokens."""
    size, keep = int(mask["size"]), int(mask.get("keep_first", 0))
    return [j for j in range(i + 1) if i - j < size or j < keep]


# ------------------------------------------------------------------ short convolution
def short_conv(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), nothing before t = 0."""
    y = torch.zeros_like(u)
    K = w.shape[1]
    for t in range(u.shape[0]):
        for j in range(K):
            at = t - K + 1 + j
            if at >= 0:
                y[t] += w[:, j] * u[at]
    return y


# ------------------------------------------------------------------ differential attention
def diff_lambda(t, p, diff):
    return torch.exp((t[p + "lq1"] * t[p + "lk1"]).sum()) - torch.exp((t[p + "lq2"] * t[p + "lk2"]).sum()) + diff


def diff_keys_values(h, t, p, mx):
    """(keys [T, G, 2, D] after convolution and rotation, values [T, G, V] after convolution)."""
    T, G, D, V = h.shape[0], mx["kv_heads"], mx["dim"], mx["vdim"]
    k = short_conv(h @ t[p + "k"].T, t[p + "k.conv"]).view(T, G, 2, D)
    v = short_conv(h @ t[p + "v"].T, t[p + "v.conv"]).view(T, G, V)
    return rotate(k, range(T), mx["rot"], True), v


def diff_attention(h, t, p, mx, eps, kept=None, layer=None):
    """kept: dict layer -> (keys, values) of the layers before; this layer's own are added."""
    T, H, G, D, V = h.shape[0], mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = short_conv(h @ t[p + "q"].T, t[p + "q.conv"]).view(T, H, 2, D)
    q = rotate(q, range(T), mx["rot"], True)
    if mx.get("kv_from") is not None:
        k, v = kept[mx["kv_from"]]
    else:
        k, v = diff_keys_values(h, t, p, mx)
        if kept is not None:
            kept[layer] = (k, v)
    lam = diff_lambda(t, p, float(mx["diff"]))
    out = torch.zeros(T, H, V, dtype=h.dtype)
    for s in range(T):
        js = visible(s, mx["mask"])
        for hd in range(H):
            g = hd // (H // G)
            a = []
            for m in range(2):
                w = torch.softmax((k[js, g, m] @ q[s, hd, m]) * float(mx["scale"]), 0)
                a.append((w[:, None] * v[js, g]).sum(0))
            out[s, hd] = rms(a[0] - lam * a[1], eps) * (1.0 - float(mx["diff"]))
    return out.reshape(T, H * V) @ t[p + "o"].T


# ------------------------------------------------------------------ latent attention
def latent_attention(h, t, p, mx, eps):
    H, D, Rd, V, rank = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
    T = h.shape[0]
    q = (h @ t[p + "q"].T).view(T, H, D + Rd)
    q_rot = rotate(q[:, :, D:], range(T), mx["rot"], False)
    dkv = h @ t[p + "dkv"].T
    c = rms(dkv[:, :rank], eps) * t[p + "dkv.norm"]
    k_rot = rotate(dkv[:, rank:], range(T), mx["rot"], False)
    k = (c @ t[p + "uk"].T).view(T, H, D)
    v = (c @ t[p + "uv"].T).view(T, H, V)
    out = torch.zeros(T, H, V, dtype=h.dtype)
    for s in range(T):
        js = visible(s, mx["mask"])
        for hd in range(H):
            sc = (k[js, hd] @ q[s, hd, :D] + k_rot[js] @ q_rot[s, hd]) * float(mx["scale"])
            out[s, hd] = (torch.softmax(sc, 0)[:, None] * v[js, hd]).sum(0)
    return out.reshape(T, H * V) @ t[p + "o"].T


# ------------------------------------------------------------------ the two parallel mixers
def normed_attention(h, t, p, mx, eps):
    H, G, D, V = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    T = h.shape[0]
    q = rms((h @ t[p + "q"].T).view(T, H, D), eps) * t[p + "q.norm"]
    k = rms((h @ t[p + "k"].T).view(T, G, D), eps) * t[p + "k.norm"]
    v = (h @ t[p + "v"].T).view(T, G, V)
    q, k = rotate(q, range(T), mx["rot"], True), rotate(k, range(T), mx["rot"], True)
    out = torch.zeros(T, H, V, dtype=h.dtype)
    for s in range(T):
        js = visible(s, mx["mask"])
        for hd in range(H):
            g = hd // (H // G)
            w = torch.softmax((k[js, g] @ q[s, hd]) * float(mx["scale"]), 0)
            out[s, hd] = (w[:, None] * v[js, g]).sum(0)
    return out.reshape(T, H * V) @ t[p + "o"].T


def gated_linear_attention(h, t, p, mx, eps):
    H, D, V, tau = mx["heads"], mx["dim"], mx["vdim"], float(mx["tau"])
    T = h.shape[0]
    q = (h @ t[p + "q"].T).view(T, H, D) * D ** -0.5
    k = (h @ t[p + "k"].T).view(T, H, D)
    v = (h @ t[p + "v"].T).view(T, H, V)
    z = (h @ t[p + "a1"].T) @ t[p + "a2"].T + t[p + "a2.b"]
    alpha = (torch.sigmoid(z) ** (1.0 / tau)).view(T, H, D)
    gate = silu(h @ t[p + "g"].T).view(T, H, V)
    out = torch.zeros(T, H, V, dtype=h.dtype)
    for hd in range(H):
        S = torch.zeros(D, V, dtype=h.dtype)
        for s in range(T):
            S = alpha[s, hd][:, None] * S + k[s, hd][:, None] * v[s, hd][None, :]
            out[s, hd] = rms(S.T @ q[s, hd], eps) * t[p + "norm"]
    return (out * gate).reshape(T, H * V) @ t[p + "o"].T


def parallel(h, t, p, mx, eps):
    return float(mx["left_scale"]) * normed_attention(h, t, p + "left.", mx["left"], eps) \
        + float(mx["right_scale"]) * gated_linear_attention(h, t, p + "right.", mx["right"], eps)


# ------------------------------------------------------------------ feed-forward
def gated_unit(h, t, p):
    return (silu(h @ t[p + "gate"].T) * (h @ t[p + "up"].T)) @ t[p + "down"].T


def router_choice(h, t, p, mlp):
    """Per token: (chosen experts, their weights)."""
    r = mlp["router"]
    E, top, count, keep = r["experts"], r["top"], r["groups"]["count"], r["groups"]["keep"]
    s = torch.softmax(h @ t[p + "router"].T, -1)
    per = E // count
    ids, wts = [], []
    for row in s:
        order = sorted(range(count), key=lambda g: -float(row[g * per:(g + 1) * per].max()))
        ok = [e for g in order[:keep] for e in range(g * per, (g + 1) * per)]
        best = sorted(ok, key=lambda e: -float(row[e]))[:top]
        w = row[best]
        ids.append(best)
        wts.append(w / (w.sum() + 1e-20) * float(r["scale"]))
    return ids, wts


def mixture(h, t, p, mlp):
    ids, wts = router_choice(h, t, p, mlp)
    out = torch.zeros_like(h)
    for s in range(h.shape[0]):
        for e, w in zip(ids[s], wts[s]):
            out[s] += w * gated_unit(h[s:s + 1], t, p + "e%d." % e)[0]
    if mlp.get("shared"):
        out = out + gated_unit(h, t, p + "shared.")
    return out


# ------------------------------------------------------------------ model
def forward(config, t, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one sequence run from position 0; layers_out receives the sum of the
    streams after every layer."""
    t = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in t.items()}
    eps = float(config["norm"]["eps"])
    x = t["embed"][torch.tensor(tokens)] * float(config["embedding"]["scale"])
    X = [x.clone() for _ in range(int(config["streams"]))]
    kept = {}
    for i, L in enumerate(config["layers"]):
        p = "l%d." % i
        h = dynamic_tanh(read_streams(X, t[p + "hc1.in"]), t, p + "norm1")
        if L["type"] == "attention":
            y = diff_attention(h, t, p + "mix.", L["mixer"], eps, kept, i)
        else:
            y = {"latent_attention": latent_attention, "parallel": parallel}[L["type"]](
                h, t, p + "mix.", L["mixer"], eps)
        X = write_streams(X, t[p + "hc1.mix"], t[p + "hc1.out"], y)
        if L.get("mlp"):
            h = dynamic_tanh(read_streams(X, t[p + "hc2.in"]), t, p + "norm2")
            X = write_streams(X, t[p + "hc2.mix"], t[p + "hc2.out"], mixture(h, t, p + "mlp.", L["mlp"]))
        if layers_out is not None:
            layers_out.append(sum(X))
    return dynamic_tanh(sum(X), t, "final.norm") @ t["head"].T
