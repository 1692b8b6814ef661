"""A plain float64 forward of the Genetar design, one function per mechanism.

TEST INFRASTRUCTURE. Whole sequences, no cache: what the device decoder's layers and caches are
compared with. It shares nothing with the product: it takes a configuration (a dict with the keys of
config.json) and a dict of tensors by name, as numpy arrays.
"""
from __future__ import annotations

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def unit_rms(x, eps):
    """x over its root mean square along the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def soft_cap(s, cap):
    return cap * np.tanh(s / cap) if cap else s


def embed_pairs(tokens, table, pairs, mul_prev, mul_cur):
    """A token's own row and one for it and the token before; the last row of `pairs` for a first token."""
    buckets = pairs.shape[0] - 1
    rows = [buckets if i == 0 else (int(tokens[i - 1]) * mul_prev + int(t) * mul_cur) % buckets for i, t in enumerate(tokens)]
    return table[np.asarray(tokens)] + pairs[rows]


def frequencies(rot):
    """Radians a position of each pair; long wavelengths are stretched where the configuration says so."""
    out = []
    for i in range(rot["dims"] // 2):
        f = rot["base"] ** (-2.0 * i / rot["dims"])
        sc = rot.get("scaling")
        if sc:
            length = 2 * np.pi / f
            if length > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif length >= sc["original"] / sc["high"]:
                s = (sc["original"] / length - sc["low"]) / (sc["high"] - sc["low"])
                f = (1 - s) * f / sc["factor"] + s * f
        out.append(f)
    return np.array(out)


def rotate_halves(x, positions, rot):
    """x [n, heads, dim]: feature i < dims / 2 turns with feature i + dims / 2; those from dims on stay."""
    half = rot["dims"] // 2
    ang = positions[:, None, None] * frequencies(rot)
    u, v = x[..., :half], x[..., half:2 * half]
    return np.concatenate([u * np.cos(ang) - v * np.sin(ang), v * np.cos(ang) + u * np.sin(ang), x[..., 2 * half:]], axis=-1)


def softmax_attend(q, k, v, scale, cap):
    """q [n, H, d], k [n, G, d], v [n, G, e], causal; H / G neighbouring query heads read one key head."""
    n, heads = q.shape[:2]
    group = heads // k.shape[1]
    out = np.empty((n, heads, v.shape[2]))
    seen = np.tril(np.ones((n, n), bool))
    for a in range(heads):
        s = soft_cap(q[:, a] @ k[:, a // group].T * scale, cap)
        s = np.where(seen, s, -np.inf)
        p = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, a] = p / p.sum(axis=1, keepdims=True) @ v[:, a // group]
    return out


def attention(h, t, mx, eps, first, unit_qk, rot, gated):
    """One attention layer. `first` is the values of the first layer that mixes values, None while there is none yet;
    returns the result and this layer's own contribution to it (its values before mixing, if it mixes)."""
    n = h.shape[0]
    q = (h @ t["q"].T).reshape(n, mx["heads"], mx["dim"])
    k = (h @ t["k"].T).reshape(n, mx["kv_heads"], mx["dim"])
    own = v = (h @ t["v"].T).reshape(n, mx["kv_heads"], mx["vdim"])
    if unit_qk:
        q, k = unit_rms(q, eps), unit_rms(k, eps)
    if rot:
        q, k = rotate_halves(q, np.arange(n), rot), rotate_halves(k, np.arange(n), rot)
    if mx["v_mix"] and first is not None:
        v = (1 - t["vmix"]) * v + t["vmix"] * first
    o = softmax_attend(q, k, v, mx["scale"], mx["softcap"])
    if gated:
        o = o * sigmoid(h @ t["g"].T)[:, :, None]
    return o.reshape(n, -1) @ t["o"].T, own if mx["v_mix"] and first is None else first


def gated_mlp(h, t):
    return (silu(h @ t["gate"].T) * (h @ t["up"].T)) @ t["down"].T


def sub(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def forward(config, tensors, tokens, streams=None):
    """Logits [n, vocab] of every position; `streams`, if a list, receives the residual after every layer."""
    t = {k: np.asarray(v, np.float64) for k, v in tensors.items()}
    eps, big = config["norm"]["eps"], config["embedding"]["bigram"]
    x = embed_pairs(tokens, t["embed"], t["bigram"], big["mul_prev"], big["mul_cur"])
    first = None
    for i, layer in enumerate(config["layers"]):
        p, mx, turned = f"l{i}.", layer["mixer"], layer["type"] == "attention_2"
        h = unit_rms(x, eps) * t[p + "norm1"]
        o, first = attention(h, sub(t, p + "mix."), mx, eps, first, unit_qk=not turned, rot=mx["rot"] if turned else None, gated=turned)
        add = o * t[p + "ls1"]
        if layer["mlp"] is not None:
            add = add + gated_mlp(h, sub(t, p + "mlp.")) * t[p + "ls2"]
        x = x + add
        if streams is not None:
            streams.append(x)
    return unit_rms(x, eps) * t["final.norm"] @ t["head"].T * config["logit_scale"]
