"""A plain float64 forward of the Fuvolix design, one function per mechanism.

TEST INFRASTRUCTURE. Whole sequences, token by token where the design is a recurrence, no cache and
no chunks: what the device decoder's layers, caches and states are compared with. It shares nothing
with the product: it takes a configuration (a dict with the keys of config.json) and a dict of
tensors by name, as numpy arrays.
"""
from __future__ import annotations

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def logsigmoid(z):
    return np.minimum(z, 0.0) - np.log1p(np.exp(-np.abs(z)))


def rms(x, eps):
    """x over its root mean square along the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def group_norm(x, w, groups, eps):
    """`groups` equal parts of the last axis, each over its own root mean square, times w."""
    parts = x.reshape(x.shape[:-1] + (groups, x.shape[-1] // groups))
    return rms(parts, eps).reshape(x.shape) * w


def causal_conv(h, w):
    """Per channel c: sum_j w[c, j] h[t - taps + 1 + j, c], zeros before the start."""
    taps = w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, h.shape[1])), h])
    return sum(padded[j:j + h.shape[0]] * w[:, j] for j in range(taps))


def rotate(x, positions, base):
    """Interleaved pairs of the whole last axis; positions along the first."""
    d = x.shape[-1]
    freq = base ** (-2.0 * np.arange(d // 2) / d)
    ang = positions[:, None] * freq
    ang = ang.reshape((x.shape[0],) + (1,) * (x.ndim - 2) + (d // 2,))
    u, v = x[..., 0::2], x[..., 1::2]
    out = np.empty_like(x)
    out[..., 0::2] = u * np.cos(ang) - v * np.sin(ang)
    out[..., 1::2] = v * np.cos(ang) + u * np.sin(ang)
    return out


def latent_attention(h, t, mx, eps):
    n, heads, dim, rd, vd, rank = h.shape[0], mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
    pos = np.arange(n)
    q = (h @ t["q"].T).reshape(n, heads, dim + rd)
    qu, qr = q[..., :dim], rotate(q[..., dim:], pos, mx["rot"]["base"])
    low = h @ t["dkv"].T
    c = rms(low[:, :rank], eps) * t["dkv.norm"]
    kr = rotate(low[:, rank:], pos, mx["rot"]["base"])
    ku = (c @ t["uk"].T).reshape(n, heads, dim)
    v = (c @ t["uv"].T).reshape(n, heads, vd)
    out = np.empty((n, heads, vd))
    for a in range(heads):
        s = (qu[:, a] @ ku[:, a].T + qr[:, a] @ kr.T) * mx["scale"]
        s = np.where(np.tril(np.ones((n, n), bool)), s, -np.inf)
        p = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, a] = (p / p.sum(axis=1, keepdims=True)) @ v[:, a]
    return out.reshape(n, heads * vd) @ t["o"].T


def mlstm_scan(q, k, v, i, f):
    """The stabilized matrix memory: q (scaled), k [n, H, d], v [n, H, e], log gates i, f [n, H] -> [n, H, e]."""
    n, heads, d = q.shape
    S, z, m = np.zeros((heads, d, v.shape[2])), np.zeros((heads, d)), np.zeros(heads)
    out = np.empty(v.shape)
    for t in range(n):
        new = np.maximum(f[t] + m, i[t])
        keep, take = np.exp(f[t] + m - new), np.exp(i[t] - new)
        m = new
        S = keep[:, None, None] * S + take[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        z = keep[:, None] * z + take[:, None] * k[t]
        num = np.einsum("hde,hd->he", S, q[t])
        den = np.maximum(np.abs(np.sum(z * q[t], axis=1)), np.exp(-m)) + 1e-6
        out[t] = num / den[:, None]
    return out


def mlstm_gates(h, t, cap):
    i = cap * np.tanh((h @ t["i"].T + t["i.b"]) / cap)
    f = logsigmoid(cap * np.tanh((h @ t["f"].T + t["f.b"]) / cap))
    return i, f


def mlstm(h, t, mx, eps):
    n, heads, dim, vd = h.shape[0], mx["heads"], mx["dim"], mx["vdim"]
    q = (h @ t["q"].T).reshape(n, heads, dim) * dim ** -0.5
    k = (h @ t["k"].T).reshape(n, heads, dim)
    v = (h @ t["v"].T).reshape(n, heads, vd)
    o = mlstm_scan(q, k, v, *mlstm_gates(h, t, mx["gate_cap"]))
    o = rms(o, eps).reshape(n, heads * vd) * t["norm"] * sigmoid(h @ t["g"].T)
    return o @ t["o"].T


def lightning_scan(q, k, v, decay):
    """S <- decay S + k v^T, o = S^T q, per head."""
    n, heads, d = q.shape
    S = np.zeros((heads, d, v.shape[2]))
    out = np.empty(v.shape)
    for t in range(n):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hde,hd->he", S, q[t])
    return out


def lightning(h, t, mx, eps):
    n, heads, dim, vd = h.shape[0], mx["heads"], mx["dim"], mx["vdim"]
    q = silu(h @ t["q"].T).reshape(n, heads, dim)
    k = silu(h @ t["k"].T).reshape(n, heads, dim)
    v = silu(h @ t["v"].T).reshape(n, heads, vd)
    o = lightning_scan(q, k, v, np.asarray(mx["decay"], float)).reshape(n, heads * vd)
    o = rms(o, eps) * t["norm"] * sigmoid(h @ t["g"].T)
    return o @ t["o"].T


MIXERS = {"latent_attention": latent_attention, "mlstm": mlstm, "lightning": lightning}


def relu2_mlp(h, t):
    return np.maximum(h @ t["up"].T, 0.0) ** 2 @ t["down"].T


def sub(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def forward(config, tensors, tokens, streams=None):
    """Logits [n, vocab] of every position; `streams`, if a list, receives the residual after every layer."""
    t = {k: np.asarray(v, np.float64) for k, v in tensors.items()}
    groups, eps = config["norm"]["groups"], config["norm"]["eps"]
    norm = lambda x, name: group_norm(x, t[name], groups, eps)
    x = norm(t["embed"][np.asarray(tokens)], "embed.norm")
    past = [x]
    for i, layer in enumerate(config["layers"]):
        p = f"l{i}."
        h = norm(x, p + "norm1")
        h = h + causal_conv(h, t[p + "canon1"])
        x = x + norm(MIXERS[layer["type"]](h, sub(t, p + "mix."), layer["mixer"], eps), p + "norm1b")
        if layer["mlp"] is not None:
            x = x + norm(relu2_mlp(norm(x, p + "norm2"), sub(t, p + "mlp.")), p + "norm2b")
        past.append(x)
        x = sum(w * y for w, y in zip(t[p + "dwa"], past))
        if streams is not None:
            streams.append(x)
    return norm(x, "final.norm") @ t["embed"].T
