"""Small Fuvolix models for the tests: configurations, random weights, and the folder a model is loaded from."""
import json
import os
import struct

import numpy as np


def latent(heads=3, dim=16, rot_dim=8, vdim=24, kv_rank=40, scale=None, base=500.0, ff=None):
    mx = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, scale=(dim + rot_dim) ** -0.5 if scale is None else scale,
              rot=dict(base=base, dims=rot_dim))
    return dict(type="latent_attention", mixer=mx, mlp=None if ff is None else dict(kind="dense", ff=ff))


def mlstm(heads=3, dim=16, vdim=24, gate_cap=9.0, ff=None):
    return dict(type="mlstm", mixer=dict(heads=heads, dim=dim, vdim=vdim, gate_cap=gate_cap), mlp=None if ff is None else dict(kind="dense", ff=ff))


def lightning(heads=3, dim=16, vdim=24, decay=None, ff=None):
    decay = list(np.linspace(0.6, 1.0, heads)) if decay is None else decay
    return dict(type="lightning", mixer=dict(heads=heads, dim=dim, vdim=vdim, decay=decay), mlp=None if ff is None else dict(kind="dense", ff=ff))


def config(layers, width=96, vocab=130, groups=3, taps=3, eps=1e-5):
    return dict(architecture="Fuvolix", width=width, vocab=vocab, canon=dict(taps=taps), norm=dict(groups=groups, eps=eps), layers=layers)


def shapes(c):
    W, out = c["width"], {"embed": (c["vocab"], c["width"]), "embed.norm": (c["width"],), "final.norm": (c["width"],)}
    for i, l in enumerate(c["layers"]):
        p, mx, H = f"l{i}.", l["mixer"], l["mixer"]["heads"]
        m = p + "mix."
        out |= {p + "norm1": (W,), p + "norm1b": (W,), p + "canon1": (W, c["canon"]["taps"]), p + "dwa": (i + 2,), m + "o": (W, H * mx["vdim"])}
        if l["mlp"]:
            out |= {p + "norm2": (W,), p + "norm2b": (W,), p + "mlp.up": (l["mlp"]["ff"], W), p + "mlp.down": (W, l["mlp"]["ff"])}
        if l["type"] == "latent_attention":
            r = mx["kv_rank"]
            out |= {m + "q": (H * (mx["dim"] + mx["rot_dim"]), W), m + "dkv": (r + mx["rot_dim"], W), m + "dkv.norm": (r,), m + "uk": (H * mx["dim"], r),
                    m + "uv": (H * mx["vdim"], r)}
        else:
            out |= {m + "q": (H * mx["dim"], W), m + "k": (H * mx["dim"], W), m + "v": (H * mx["vdim"], W), m + "g": (H * mx["vdim"], W),
                    m + "norm": (H * mx["vdim"],)}
            if l["type"] == "mlstm":
                out |= {m + "i": (H, W), m + "f": (H, W), m + "i.b": (H,), m + "f.b": (H,)}
    return out


def to_bf16(x):
    """The nearest bfloat16 (ties to even), as float32."""
    b = np.asarray(x, np.float32).view(np.uint32)
    return ((b + 0x7fff + ((b >> 16) & 1)) & np.uint32(0xffff0000)).view(np.float32)


def weights(c, seed=0):
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in shapes(c).items():
        leaf = name.rsplit(".", 1)[-1]
        w = rng.normal(size=shape)
        if "norm" in leaf:
            w = 1 + 0.3 * w
        elif leaf == "canon1":
            w = w * 0.5
        elif leaf == "dwa":
            w = 0.4 * w + 0.3
        elif name.endswith("f.b"):
            w = 3 + w
        elif leaf not in ("embed", "b"):
            w = w / np.sqrt(shape[-1])
        out[name] = to_bf16(w)
    return out


def write(folder, c, tensors):
    """config.json and model.safetensors."""
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(c, f)
    index, blobs, at = {}, [], 0
    for name, w in tensors.items():
        raw = (np.ascontiguousarray(w, np.float32).view(np.uint32) >> 16).astype("<u2").tobytes()
        index[name] = dict(dtype="BF16", shape=list(w.shape), data_offsets=[at, at + len(raw)])
        blobs.append(raw)
        at += len(raw)
    head = json.dumps(index).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(head)) + head + b"".join(blobs))
    return str(folder)


def tokens(c, n, seed=0, batch=None):
    rng = np.random.default_rng(1000 + seed)
    return rng.integers(0, c["vocab"], n if batch is None else (batch, n)).astype(np.int32)


def error(got, want, quantile=1.0):
    """A row's error: root mean square over the vocabulary with the mean taken off, over that of all the wanted logits. The
    largest, or another quantile of the rows'."""
    d = np.asarray(got, np.float64) - want
    d = d - d.mean(axis=-1, keepdims=True)
    spread = want - want.mean(axis=-1, keepdims=True)
    return float(np.quantile(np.sqrt((d * d).mean(axis=-1)), quantile) / np.sqrt((spread * spread).mean()))
