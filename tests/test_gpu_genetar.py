"""The Genetar decoder on a real MI355X against the plain float64 forward: every mechanism alone and together, in both
compute dtypes, in whole prompts, portions and decoding, through the registry, the handle and the greedy loop."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from mimir_amd import capi, registry, stack
from oracle import fuvolix as F
from oracle import genetar as G
from tests import genetar as X
from tests import gpu

pytestmark = pytest.mark.gpu

DTYPES = ("float32", "bfloat16")
# of a row's logits, against the spread of all of them (tests.fuvolix.error)
TOL = {"float32": 1e-5, "bfloat16": 0.03}
off = lambda t: t * 0


def load(folder, c, w, context=256, dtype="float32", **kw):
    gpu.lib()
    return registry.load(X.write(folder, c, w), context=context, dtype=dtype, **kw)


def in_portions(m, toks, sizes):
    """Every position's logits, the tokens in portions of these sizes (repeated)."""
    m.reset()
    out, at, i = [], 0, 0
    while at < len(toks):
        n = min(sizes[i % len(sizes)], len(toks) - at)
        out.append(m.logits_at(toks[at:at + n], range(n)))
        at, i = at + n, i + 1
    assert m.cache_len == len(toks)
    return np.concatenate(out)


def changed(w, **leaves):
    """w with every tensor whose name ends with a leaf replaced by fn(tensor)."""
    out = dict(w)
    for leaf, fn in leaves.items():
        hit = [k for k in w if k.endswith("." + leaf) or k == leaf]
        assert hit, leaf
        for k in hit:
            out[k] = X.to_bf16(fn(w[k]))
    return out


def _mechanisms():
    """One mechanism of the design at a time: what else there is is switched off by its weights."""
    plain = dict(bigram=off)
    yield "pairs_of_tokens", X.config([X.unit()]), dict(o=off, embed=lambda t: 0.2 * t)
    yield "one_bucket", X.config([X.unit()], buckets=1, mul_prev=1, mul_cur=1), dict(o=off, embed=lambda t: 0.2 * t)
    yield "large_multipliers", X.config([X.unit()], buckets=101, mul_prev=2 ** 31 - 1, mul_cur=2 ** 31 - 3), dict(o=off, embed=lambda t: 0.2 * t)
    yield "feed_forward", X.config([X.unit(ff=200), X.unit(ff=71)]), dict(plain, o=off)
    yield "no_feed_forward", X.config([X.unit()]), plain
    yield "scales_of_nothing", X.config([X.unit(ff=72), X.rotary(ff=40)]), dict(plain, ls2=lambda t: t * (np.arange(80) % 3 > 0), ls1=lambda t: t * (np.arange(80) % 4 > 0))
    yield "scales_far_apart", X.config([X.unit(ff=72), X.rotary(ff=40)]), dict(plain, ls2=lambda t: t * 10.0 ** -(np.arange(80) % 5))
    yield "scales_of_one", X.config([X.unit(ff=72)]), dict(plain, ls2=lambda t: t * 0 + 1, ls1=lambda t: t * 0 + 1)
    yield "unit_queries_and_keys", X.config([X.unit(v_mix=False)]), dict(plain, q=lambda t: t * np.repeat(4.0 ** np.arange(6), 24)[:, None])
    yield "eps_of_small_keys", X.config([X.unit(v_mix=False)], eps=0.02), dict(plain, k=lambda t: t * 0.1, q=lambda t: t * 0.3)
    yield "rotation", X.config([X.rotary(v_mix=False, softcap=1e4)]), dict(plain, g=lambda t: t * 0)
    yield "rotation_of_all", X.config([X.rotary(v_mix=False, rot=24, base=1e4, low=1.0, high=4.0, original=8192, factor=8.0)]), plain
    yield "rotation_scaled_all", X.config([X.rotary(v_mix=False, rot=8, base=5.0, low=90.0, high=100.0, original=64, factor=2.0)]), plain
    yield "rotation_scaled_between", X.config([X.rotary(v_mix=False, rot=12, base=40.0, low=0.01, high=50.0, original=100, factor=6.0)]), plain
    yield "gate", X.config([X.rotary(v_mix=False)]), dict(plain, g=lambda t: t * 4)
    yield "sharp_cap", X.config([X.unit(v_mix=False, softcap=1.5, scale=1.0)]), plain
    yield "cap_with_running_maximum", X.config([X.unit(v_mix=False, softcap=50.0, scale=2.0)]), plain
    yield "no_cap", X.config([X.unit(v_mix=False, softcap=None, scale=2.0)]), plain
    yield "values_mixed", X.config([X.unit(v_mix=False), X.unit(), X.rotary(v_mix=False), X.rotary(), X.unit()]), plain
    yield "values_of_the_first_only", X.config([X.unit(), X.unit(), X.rotary()]), dict(plain, vmix=lambda t: t * 0 + 1)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,c,edits", list(_mechanisms()), ids=[m[0] for m in _mechanisms()])
def test_mechanism_alone(tmp_path, name, c, edits, dtype):
    w = changed(X.weights(c, 1), **edits)
    toks = X.tokens(c, 150)
    want = G.forward(c, w, toks)
    gpu.say(f"genetar {name} {dtype}")
    m = load(tmp_path, c, w, dtype=dtype)
    errs = {"whole": X.error(in_portions(m, toks, [150]), want), "portions": X.error(in_portions(m, toks, [70, 3, 9]), want),
            "single": X.error(in_portions(m, toks, [1]), want)}
    print(name, dtype, errs)
    assert max(errs.values()) < TOL[dtype]


MIX = [X.rotary(ff=200, v_mix=False), X.unit(ff=136), X.rotary(heads=6, kv_heads=2, dim=40, vdim=16, rot=16, softcap=40.0), X.unit(heads=4, kv_heads=4, dim=16, vdim=8, ff=64, v_mix=False),
       X.unit(heads=2, kv_heads=2, dim=72, vdim=16), X.rotary(heads=10, kv_heads=2, dim=8, rot=2)]


@pytest.fixture(scope="module")
def mixed(tmp_path_factory):
    """A model of layers that differ in everything, its tokens, and every position's logits from the plain forward."""
    c = X.config(MIX, width=128, buckets=301, mul_prev=77, mul_cur=3)
    w = X.weights(c, 2)
    toks = X.tokens(c, 210)
    return c, w, toks, G.forward(c, w, toks), X.write(tmp_path_factory.mktemp("mixed"), c, w)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [[210], [1], [2], [3, 2], [9, 1], [16], [31, 33, 2], [63, 1, 65, 64], [128, 7], [100, 2, 2]], ids=str)
def test_portions(mixed, sizes, dtype):
    """Cut anywhere, at and around the kernels' own tiles (64, 128) and thresholds (8, 32), the logits are those of the
    whole prompt."""
    c, w, toks, want, folder = mixed
    gpu.say(f"genetar portions {sizes} {dtype}")
    m = registry.load(folder, context=210, dtype=dtype)
    e = X.error(in_portions(m, toks, sizes), want)
    print(sizes, dtype, e)
    assert e < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_sequence(mixed, dtype):
    """Several shares of the keys, many tiles, and decoding far behind a long prompt."""
    c, w, _, _, folder = mixed
    toks = X.tokens(c, 1100, 3)
    want = G.forward(c, w, toks)
    gpu.say(f"genetar long {dtype}")
    m = registry.load(folder, context=1300, dtype=dtype)
    for sizes in ([1100], [1030, 1, 20, 1], [513, 40]):
        e = X.error(in_portions(m, toks, sizes), want)
        print(sizes, dtype, e)
        assert e < TOL[dtype], sizes


@pytest.mark.parametrize("dtype", DTYPES)
def test_calls_longer_than_a_pass(mixed, dtype):
    """A call of more tokens than the activations hold runs in several passes; wanted rows in any order, also repeated."""
    c, w, toks, want, folder = mixed
    gpu.say(f"genetar passes {dtype}")
    m = registry.load(folder, context=210, max_tokens=48, dtype=dtype)
    ask = [209, 0, 47, 48, 48, 95, 96, 150, 1]
    assert X.error(m.logits_at(toks, ask), want[ask]) < TOL[dtype]
    m.reset()
    assert m.logits_at(toks[:100], []).shape == (0, c["vocab"])
    assert X.error(m.logits_at(toks[100:], [0, 109]), want[[100, 209]]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_sequences_in_lockstep_and_slots_used_again(mixed, dtype):
    """Three sequences at once against each alone; then the same slots for shorter ones: nothing of the sequence before is left."""
    c, w, _, _, folder = mixed
    gpu.say(f"genetar batch {dtype}")
    t3 = X.tokens(c, 90, 5, batch=3)
    want = np.stack([G.forward(c, w, t) for t in t3])
    m = registry.load(folder, context=128, batch=3, dtype=dtype)
    for again in range(2):
        m.reset()
        a = m.logits(t3[:, :70], all=True)
        b = [m.logits(t3[:, t:t + 1]) for t in range(70, 80)]  # rows of one position each
        z = m.logits(t3[:, 80:], all=True)
        got = np.concatenate([a, np.stack(b, 1), z], 1)
        assert X.error(got, want) < TOL[dtype]
    short = X.tokens(c, 3, 9, batch=3)
    m.reset()
    assert X.error(m.logits(short, all=True), np.stack([G.forward(c, w, t) for t in short])) < TOL[dtype]
    one = registry.load(folder, context=128, dtype=dtype)
    assert X.error(one.logits(t3[1], all=True)[0], got[1]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_first_tokens_of_a_sequence(mixed, dtype):
    c, w, toks, want, folder = mixed
    gpu.say(f"genetar first tokens {dtype}")
    m = registry.load(folder, context=64, dtype=dtype)
    for n in (1, 2, 3, 5, 9, 17, 33, 64):
        m.reset()
        assert X.error(m.logits(toks[:n], all=True)[0], want[:n]) < TOL[dtype], n


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("place", [0, 1, 15, 16, 63, 64, 65, 127, 128, 300])
@pytest.mark.parametrize("kind", ["unit", "rotary"])
def test_one_far_key_stands_out(tmp_path, kind, place, dtype):
    """One token that no other position has, whose key a sharp query finds among hundreds: the rows that see it differ
    from those of a sequence without it by far more than the tolerance, and agree with the plain forward."""
    layer = X.unit(heads=4, kv_heads=2, dim=32, vdim=32, scale=0.9, softcap=25.0, v_mix=False) if kind == "unit" else \
        X.rotary(heads=4, kv_heads=2, dim=32, vdim=32, scale=0.9, softcap=35.0, v_mix=False, rot=8)
    c = X.config([layer], width=64, vocab=80)
    w = changed(X.weights(c, 3), bigram=off, norm1=lambda t: t * 0 + 1, ls1=lambda t: 3 * t)
    rng = np.random.default_rng(4)
    # tokens 0..77 are ordinary; 78 is the key (features 0..15, which keys are made of) and 79 asks (48..63, which queries
    # are made of)
    e = w["embed"].copy()
    e[:78, :16] = 0.1 * rng.normal(size=(78, 16))
    e[:78, 48:] = 0.1 * rng.normal(size=(78, 16))
    e[78], e[79] = 0, 0
    e[78, :16], e[78, 16:48] = 3, rng.normal(size=32)
    e[79, 48:], e[79, 16:48] = 3, rng.normal(size=32)
    w["embed"] = X.to_bf16(e)
    toks = rng.integers(0, 78, 333).astype(np.int32)
    toks[-1] = toks[place + 1] = 79
    without = toks.copy()
    toks[place] = 78
    # every head's queries and keys meet in features 16 .., which do not turn
    q, k = w["l0.mix.q"] * 0.05, w["l0.mix.k"] * 0.05
    for h in range(4):
        q[h * 32 + 16 + np.arange(16), 48 + np.arange(16)] = 0.5
    for h in range(2):
        k[h * 32 + 16 + np.arange(16), np.arange(16)] = 0.5
    w |= {"l0.mix.q": X.to_bf16(q), "l0.mix.k": X.to_bf16(k)}
    want = G.forward(c, w, toks)
    apart = X.error(G.forward(c, w, without)[-1:], want[-1:])
    assert apart > 0.25, apart  # the key is what the last row is about
    gpu.say(f"genetar far key {kind} {place} {dtype}")
    m = load(tmp_path, c, w, context=333, dtype=dtype)
    for sizes in ([333], [300, 32, 1], [100, 2, 64]):
        e = X.error(in_portions(m, toks, sizes), want)
        assert e < TOL[dtype], (sizes, e)


SIZES = {
    "odd": X.config([X.unit(heads=5, kv_heads=5, dim=10, vdim=7, ff=33), X.rotary(heads=6, kv_heads=3, dim=9, vdim=7, rot=6, v_mix=False, ff=1), X.rotary(heads=10, kv_heads=5, dim=5, vdim=7, rot=4)],
                    width=75, vocab=101, eps=1e-3, buckets=3),
    "one_of_each": X.config([X.unit(heads=1, kv_heads=1, dim=1, vdim=1, ff=1), X.rotary(heads=1, kv_heads=1, dim=2, vdim=1, rot=2)], width=32, vocab=40),
    "many_heads_a_group": X.config([X.unit(heads=19, kv_heads=1, dim=8, vdim=8), X.rotary(heads=34, kv_heads=2, dim=16, vdim=4, rot=8, v_mix=False)], width=160),
    "wide_heads": X.config([X.unit(heads=4, kv_heads=2, dim=128, vdim=128, ff=512), X.rotary(heads=2, kv_heads=1, dim=100, vdim=120, rot=64, v_mix=False)], width=256),
    "wider_heads": X.config([X.unit(heads=2, kv_heads=1, dim=192, vdim=160), X.rotary(heads=2, kv_heads=2, dim=256, vdim=80, rot=256, v_mix=False), X.unit(heads=2, kv_heads=1, dim=64, vdim=256, v_mix=False)],
                            width=192),
    "past_the_matrix_cores": X.config([X.unit(heads=2, kv_heads=1, dim=300, vdim=24), X.rotary(heads=3, kv_heads=1, dim=24, vdim=290, rot=24, v_mix=False)], width=96),
    "narrow": X.config([X.unit(heads=2, kv_heads=1, dim=8, vdim=8, ff=20)], width=16, vocab=24),
    "wide": X.config([X.unit(heads=5, kv_heads=1, dim=96, vdim=72, ff=300), X.rotary(heads=4, kv_heads=1, dim=64, vdim=72, rot=32)], width=2304),
    "long_sums": X.config([X.unit(heads=40, kv_heads=8, dim=64, vdim=64, ff=8200)], width=512),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", SIZES)
def test_other_sizes(tmp_path, name, dtype):
    c = SIZES[name]
    w = X.weights(c, 7)
    toks = X.tokens(c, 140, 7)
    want = G.forward(c, w, toks)
    gpu.say(f"genetar sizes {name} {dtype}")
    m = load(tmp_path, c, w, context=140, dtype=dtype)
    for sizes in ([140], [67, 2, 40, 1]):
        e = X.error(in_portions(m, toks, sizes), want)
        print(name, dtype, sizes, e)
        assert e < TOL[dtype], (sizes, e)


@pytest.mark.parametrize("dtype", DTYPES)
def test_large_prompt_tiles(tmp_path, dtype):
    """Products large enough for the tiles of 128 and 256 rows, with both factors, and rows that fill no tile."""
    c = X.config([X.rotary(heads=8, kv_heads=2, dim=64, vdim=64, rot=64, ff=3500), X.unit(heads=8, kv_heads=2, dim=64, vdim=64, ff=3500)], width=1280, vocab=90)
    w = X.weights(c, 9)
    toks = X.tokens(c, 530, 9, batch=8)
    one = G.forward(c, w, toks[5])
    gpu.say(f"genetar large tiles {dtype}")
    m = load(tmp_path, c, w, context=530, batch=8, dtype=dtype)
    got = m.logits(toks, all=True)[5]
    print(dtype, X.error(got, one))
    assert X.error(got, one) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("swiglu", [False, True], ids=["relu2", "swiglu"])
@pytest.mark.parametrize("bare", [False, True], ids=["posts", "bare"])
def test_attention_in_the_other_arrangement(dtype, swiglu, bare, monkeypatch):
    """The mixer, the gated feed-forward and the layers' scales in layers that run in turn, with and without norms of results,
    convolution and average."""
    mx = X.rotary(heads=4, kv_heads=2, dim=24, vdim=16, rot=10, v_mix=False)["mixer"]
    W, vocab, ff, taps = 96, 70, 56, 1 if bare else 3
    flags = capi.STACK_LAYER_SCALE if bare else capi.STACK_EMBED_NORM | capi.STACK_POST_NORMS | capi.STACK_DEPTH_AVERAGE
    sc = mx["rot"]["scaling"]
    layers = [capi.StackLayer(mixer=capi.MIXER_ATTENTION, heads=4, kv_heads=2, dim=24, vdim=16, rot_dim=10, ff=ff, mlp=capi.MLP_SWIGLU if swiglu else capi.MLP_RELU2,
                              head_gate=1, scale=mx["scale"], softcap=mx["softcap"], rot_base=mx["rot"]["base"], rot_factor=sc["factor"], rot_low=sc["low"],
                              rot_high=sc["high"], rot_original=sc["original"]) for _ in range(2)]
    config = capi.StackConfig(width=W, vocab=vocab, layers=2, context=100, batch=1, taps=0 if bare else taps, norm_groups=2, dtype=stack.DTYPES[dtype], flags=flags, eps=1e-5,
                              logit_scale=1.0)
    gpu.lib()
    m = stack.Stack(config, layers)
    rng, w = np.random.default_rng(8), {}
    for name, n, k in m.tensors():
        leaf = name.rsplit(".", 1)[-1]
        if leaf == "vmix":
            continue
        t = rng.normal(size=(n, k) if n > 1 or leaf in ("g",) else (k,))
        t = t if leaf == "embed" else t / np.sqrt(k) if n > 1 else 1 + 0.3 * t if "norm" in leaf else 0.5 + 0.4 * t
        w[name] = X.to_bf16(t.reshape(W, taps) if leaf == "canon1" else t)
        m.set_tensor(name, capi.BF16, (w[name].view(np.uint32) >> 16).astype(np.uint16), n * k)
    m.finalize(100)
    # the plain forward of layers in turn, with this mixer; what a bare stack leaves out is nothing there
    scales = iter([w.pop(f"l{i}.ls{j}").astype(np.float64) for i in range(2) for j in (1, 2)] if bare else [np.ones(W)] * 4)
    if bare:
        w |= {"embed.norm": np.ones(W)} | {f"l{i}.{n}": np.ones(W) for i in range(2) for n in ("norm1b", "norm2b")} | {f"l{i}.canon1": np.zeros((W, 1)) for i in range(2)}
        w |= {f"l{i}.dwa": np.eye(1, i + 2, i + 1)[0] for i in range(2)}
        norm = F.group_norm
        monkeypatch.setattr(F, "group_norm", lambda x, g, groups, eps: x if np.all(g == 1) else norm(x, g, groups, eps))
    monkeypatch.setitem(F.MIXERS, "attention_2", lambda h, t, mx, eps: G.attention(h, t, mx, eps, None, False, mx["rot"], True)[0] * next(scales))
    relu2 = F.relu2_mlp
    monkeypatch.setattr(F, "relu2_mlp", lambda h, t: (G.gated_mlp(h, t) if swiglu else relu2(h, t)) * next(scales))
    cfg = dict(norm=dict(groups=2, eps=1e-5), layers=[dict(type="attention_2", mixer=mx, mlp=dict(kind="dense", ff=ff))] * 2)
    toks = np.random.default_rng(2).integers(0, vocab, 90).astype(np.int32)
    want = F.forward(cfg, w, toks)
    gpu.say(f"attention in turn {dtype} swiglu {swiglu} bare {bare}")
    for sizes in ([90], [1], [40, 2, 9]):
        e = X.error(in_portions(m, toks, sizes), want)
        print(sizes, e)
        assert e < TOL[dtype], sizes


def test_greedy_generation(mixed):
    """The greedy loop (a recorded step; the same launches one by one; calls with the position from the host) in float32
    against the plain forward's choices, far into decoding. Where the two best logits are close, either may be chosen."""
    c, w, toks, _, folder = mixed
    lib = gpu.lib()
    m = registry.load(folder, context=256, dtype="float32")
    prompt, n = toks[:70], 120
    gpu.say("genetar greedy")
    runs = []
    try:
        for mode in (0, 1, 2):
            capi.check(lib.mi355x_tune(b"llama.step", mode))
            m.reset()
            out, secs = m.generate(prompt, n)
            assert secs[0] > 0 and m.cache_len == 70 + n - 1
            runs.append(out[0])
    finally:
        capi.check(lib.mi355x_tune(b"llama.step", 0))
    m.reset()
    replayed, _ = m.generate(prompt, n)  # the recorded step once more
    runs.append(replayed[0])
    for out in runs:
        lg = G.forward(c, w, np.concatenate([prompt, out]))[69:-1]
        chosen = lg[np.arange(n), out]
        assert np.all(lg.max(1) - chosen < 1e-3 * lg.std())
    # generation goes on from what the sequence holds
    more = m.logits_at([int(replayed[0, -1])], [0])
    assert X.error(more, G.forward(c, w, np.concatenate([prompt, replayed[0]]))[-1:]) < TOL["float32"]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("batch", [1, 3, 10])  # one row, a product of few rows, more than it takes
def test_generation_of_several_sequences(mixed, batch, dtype):
    """Each of the sequences chooses as it does alone (bfloat16: as long as no two logits are closer than its rounding)."""
    c, w, _, _, folder = mixed
    gpu.say(f"genetar greedy batch {batch} {dtype}")
    prompts = X.tokens(c, 40, 11, batch=batch)
    m = registry.load(folder, context=160, batch=batch, dtype=dtype)
    out, _ = m.generate(prompts, 90)
    for b in {0, batch // 2, batch - 1}:
        lg = G.forward(c, w, np.concatenate([prompts[b], out[b]]))[39:-1]
        behind = lg.max(1) - lg[np.arange(90), out[b]]
        assert np.all(behind < (1e-3 if dtype == "float32" else 0.25) * lg.std()), behind.max() / lg.std()


def test_errors_before_anything_runs(tmp_path, mixed):
    c, w, toks, _, folder = mixed
    gpu.say("genetar errors")
    m = registry.load(folder, context=20, dtype="float32")
    with pytest.raises(capi.Mi355xError) as e:
        m.logits(toks[:21])
    assert e.value.status == capi.ERR_SHAPE
    with pytest.raises(capi.Mi355xError) as e:
        m.logits([0, c["vocab"]])
    assert e.value.status == capi.ERR_INDEX
    assert m.cache_len == 0
    for name in ("l1.mix.k", "l2.mix.vmix", "l0.ls2", "bigram", "head", "l5.mix.g"):
        part = dict(w)
        del part[name]
        with pytest.raises(capi.Mi355xError, match=name):
            load(tmp_path, c, part)
    with pytest.raises(capi.Mi355xError, match="elements"):
        load(tmp_path, c, w | {"bigram": w["bigram"][:-1]})
    with pytest.raises(capi.Mi355xError, match="unknown tensor"):
        load(tmp_path, c, w | {"l1.mix.g": w["l0.mix.g"]})


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay(tmp_path, mixed, dtype):
    """bin/trace_run: requests one after the other, cut into steps; its logits are the plain forward's."""
    c, w, toks, want, folder = mixed
    steps = [dict(step=0, entries=[dict(id="a", tokens=toks[:50].tolist(), want=[0, 49])], end=[]),
             dict(step=1, entries=[dict(id="a", tokens=toks[50:52].tolist(), want=[])], end=[]),
             dict(step=2, entries=[dict(id="a", tokens=toks[52:53].tolist(), want=[0])], end=["a"]),
             dict(step=3, entries=[dict(id="b", tokens=toks[:12].tolist(), want=[11, 3])], end=["b"])]
    gpu.say(f"genetar trace {dtype}")
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out = tmp_path / "out"
    out.mkdir()
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", str(out), "--max-tokens", "64"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert r.stdout.split("\n")[:4] == [f"done {i}" for i in range(4)]
    assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "3.f32"]
    for step, rows in ((0, [0, 49]), (2, [52]), (3, [11, 3])):
        got = np.fromfile(out / f"{step}.f32", "<f4").reshape(len(rows), c["vocab"])
        assert X.error(got, want[rows]) < TOL[dtype]
