"""Small Genetar models for the tests: configurations and random weights (folders, tokens and errors as for Fuvolix)."""
import numpy as np

from tests.fuvolix import error, to_bf16, tokens, write  # noqa: F401


def _layer(kind, heads, kv_heads, dim, vdim, scale, softcap, v_mix, ff, **more):
    mx = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=dim ** -0.5 if scale is None else scale, softcap=softcap, v_mix=v_mix, **more)
    return dict(type=kind, mixer=mx, mlp=None if ff is None else dict(kind="dense", ff=ff))


def unit(heads=6, kv_heads=2, dim=24, vdim=16, scale=None, softcap=12.0, v_mix=True, ff=None):
    return _layer("attention", heads, kv_heads, dim, vdim, scale, softcap, v_mix, ff)


def rotary(heads=6, kv_heads=2, dim=24, vdim=16, scale=None, softcap=7.0, v_mix=True, ff=None, rot=10, base=300.0, factor=3.0, low=1.5, high=6.0, original=64):
    return _layer("attention_2", heads, kv_heads, dim, vdim, scale, softcap, v_mix, ff,
                  rot=dict(base=base, dims=rot, scaling=dict(factor=factor, low=low, high=high, original=original)))


def config(layers, width=80, vocab=130, eps=1e-5, buckets=37, mul_prev=11, mul_cur=5, logit_scale=0.7):
    return dict(architecture="Genetar", width=width, vocab=vocab, norm=dict(eps=eps), logit_scale=logit_scale,
                embedding=dict(bigram=dict(buckets=buckets, mul_prev=mul_prev, mul_cur=mul_cur)), layers=layers)


def shapes(c):
    W = c["width"]
    out = {"embed": (c["vocab"], W), "bigram": (c["embedding"]["bigram"]["buckets"] + 1, W), "final.norm": (W,), "head": (c["vocab"], W)}
    for i, l in enumerate(c["layers"]):
        p, mx = f"l{i}.", l["mixer"]
        m, H, G = p + "mix.", mx["heads"], mx["kv_heads"]
        out |= {p + "norm1": (W,), p + "ls1": (W,), m + "q": (H * mx["dim"], W), m + "k": (G * mx["dim"], W), m + "v": (G * mx["vdim"], W), m + "o": (W, H * mx["vdim"])}
        if mx["v_mix"]:
            out[m + "vmix"] = ()
        if l["type"] == "attention_2":
            out[m + "g"] = (H, W)
        if l["mlp"]:
            out |= {p + "ls2": (W,), p + "mlp.gate": (l["mlp"]["ff"], W), p + "mlp.up": (l["mlp"]["ff"], W), p + "mlp.down": (W, l["mlp"]["ff"])}
    return out


def weights(c, seed=0):
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in shapes(c).items():
        leaf = name.rsplit(".", 1)[-1]
        w = rng.normal(size=shape)
        if "norm" in leaf:
            w = 1 + 0.3 * w
        elif leaf in ("ls1", "ls2"):
            w = 0.8 + 0.4 * w
        elif leaf == "vmix":
            w = rng.uniform(0.1, 0.9, size=shape)
        elif leaf not in ("embed", "bigram"):
            w = w / np.sqrt(shape[-1]) * (1.6 if leaf in ("q", "k") else 1.0)
        out[name] = to_bf16(w)
    return out
