"""The Fuvolix decoder on a real MI355X against the plain float64 forward: every mechanism alone and together, in both
compute dtypes, in whole prompts, portions and decoding, through the registry, the handle and the greedy loop."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from mimir_amd import capi, registry
from oracle import fuvolix as F
from tests import fuvolix as X
from tests import gpu

pytestmark = pytest.mark.gpu

DTYPES = ("float32", "bfloat16")
# of a row's logits, against the spread of all of them (tests.fuvolix.error)
TOL = {"float32": 1e-4, "bfloat16": 0.06}
# between two ways of running the same tokens
SAME = {"float32": 1e-4, "bfloat16": 0.06}


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
    """w with every tensor whose name ends with a leaf (dots as __) replaced by fn(tensor)."""
    out = dict(w)
    for leaf, fn in leaves.items():
        hit = [k for k in w if k.endswith("." + leaf.replace("__", ".")) or k == leaf]
        assert hit, leaf
        for k in hit:
            out[k] = X.to_bf16(fn(w[k]))
    return out


off = lambda t: t * 0


def _mechanisms():
    """One mechanism of the design at a time: what else a layer has is switched off by its weights."""
    plain = dict(canon1=off, dwa=lambda t: np.eye(1, t.size, t.size - 1)[0])
    yield "group_norm", X.config([X.lightning(), X.lightning()], groups=8), dict(plain, o=off, embed=lambda t: t * np.repeat(4.0 ** np.arange(8), 12))
    yield "one_group", X.config([X.lightning()], groups=1), dict(plain, o=off)
    yield "convolution", X.config([X.lightning(decay=[0.0, 0.0, 0.0])], taps=5), {}
    yield "one_tap", X.config([X.lightning(decay=[0.0, 0.0, 0.0])], taps=1), {}
    yield "depth_average", X.config([X.lightning(heads=1, decay=[0.5]) for _ in range(11)]), dict(canon1=off)
    yield "mlp", X.config([X.lightning(ff=200), X.lightning(ff=72)]), dict(plain, o=off)
    yield "lightning", X.config([X.lightning(decay=[1.0, 0.5, 0.99])]), plain
    yield "mlstm", X.config([X.mlstm()]), plain
    yield "latent_attention", X.config([X.latent()]), plain


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,c,edits", list(_mechanisms()), ids=[m[0] for m in _mechanisms()])
def test_mechanism_alone(tmp_path, name, c, edits, dtype):
    w = changed(X.weights(c, 1), **edits)
    toks = X.tokens(c, 150)
    want = F.forward(c, w, toks)
    gpu.say(f"fuvolix {name} {dtype}")
    m = load(tmp_path, c, w, dtype=dtype)
    errs = {"whole": X.error(in_portions(m, toks, [150]), want), "portions": X.error(in_portions(m, toks, [70, 3, 9]), want),
            "single": X.error(in_portions(m, toks, [1]), want)}
    print(name, dtype, errs)
    assert max(errs.values()) < TOL[dtype]


MIX = [X.lightning(ff=200), X.latent(ff=136), X.mlstm(), X.latent(heads=2, dim=24, rot_dim=16, vdim=16, kv_rank=64, base=10.0), X.mlstm(heads=2, dim=40, vdim=8, ff=64),
       X.lightning(heads=5, dim=8, vdim=40)]


@pytest.fixture(scope="module")
def mixed(tmp_path_factory):
    """A model of all mixers, its tokens, and every position's logits from the plain forward."""
    c = X.config(MIX, width=128, groups=2, taps=4)
    w = X.weights(c, 2)
    toks = X.tokens(c, 210)
    return c, w, toks, F.forward(c, w, toks), X.write(tmp_path_factory.mktemp("mixed"), c, w)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [[210], [1], [2], [3, 2], [9, 1], [16], [31, 33, 2], [63, 1, 65, 64], [128, 7], [100, 2, 2]], ids=str)
def test_portions(mixed, sizes, dtype):
    """Cut anywhere, at and around the kernels' own chunks (64) and thresholds (8, 16, 32), the logits are those of the
    whole prompt."""
    c, w, toks, want, folder = mixed
    gpu.say(f"fuvolix portions {sizes} {dtype}")
    m = registry.load(folder, context=210, dtype=dtype)
    e = X.error(in_portions(m, toks, sizes), want)
    print(sizes, dtype, e)
    assert e < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_calls_longer_than_a_pass(mixed, dtype):
    """A call of more tokens than the activations hold runs in several passes; wanted rows in any order, also repeated."""
    c, w, toks, want, folder = mixed
    gpu.say(f"fuvolix passes {dtype}")
    m = registry.load(folder, context=210, max_tokens=48, dtype=dtype)
    ask = [209, 0, 47, 48, 48, 95, 96, 150, 1]
    assert X.error(m.logits_at(toks, ask), want[ask]) < TOL[dtype]
    m.reset()
    assert m.logits_at(toks[:100], []).shape == (0, c["vocab"])
    assert X.error(m.logits_at(toks[100:], [0, 109]), want[[100, 209]]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_sequences_in_lockstep_and_states_used_again(mixed, dtype):
    """Three sequences at once against each alone; then the same slots for shorter ones: nothing of the sequence before is left."""
    c, w, _, _, folder = mixed
    gpu.say(f"fuvolix batch {dtype}")
    t3 = X.tokens(c, 90, 5, batch=3)
    want = np.stack([F.forward(c, w, t) for t in t3])
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
    assert X.error(m.logits(short, all=True), np.stack([F.forward(c, w, t) for t in short])) < TOL[dtype]
    one = registry.load(folder, context=128, dtype=dtype)
    assert X.error(one.logits(t3[1], all=True)[0], got[1]) < SAME[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_first_tokens_of_a_sequence(mixed, dtype):
    c, w, toks, want, folder = mixed
    gpu.say(f"fuvolix first tokens {dtype}")
    m = registry.load(folder, context=64, dtype=dtype)
    for n in (1, 2, 3, 5, 9, 17):
        m.reset()
        assert X.error(m.logits(toks[:n], all=True)[0], want[:n]) < TOL[dtype], n


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("place", [0, 1, 63, 64, 65, 127, 128, 300])
def test_one_far_key_stands_out(tmp_path, place, dtype):
    """One token that no other position has, whose key a sharp query finds among hundreds: the rows that see it differ
    from those of a sequence without it by far more than the tolerance, and agree with the plain forward."""
    c = X.config([X.latent(heads=2, dim=32, rot_dim=4, vdim=32, kv_rank=64, scale=1.0, base=1e6)], width=64, vocab=80, groups=1, taps=1)
    w = changed(X.weights(c, 3), canon1=off, dkv__norm=lambda t: t * 0 + 1, dwa=lambda t: np.array([0.0, 1.0]), norm1b=lambda t: 3 * t)
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
    # both heads' queries and keys meet in the latent's first features
    q, dkv, uk = w["l0.mix.q"] * 0.1, w["l0.mix.dkv"].copy(), w["l0.mix.uk"] * 0.05
    dkv[:16, :] = 0
    dkv[np.arange(16), np.arange(16)] = 2
    for h in range(2):
        uk[h * 32:h * 32 + 16, :] = 0
        uk[h * 32 + np.arange(16), np.arange(16)] = 1
        q[h * 36 + np.arange(16), 48 + np.arange(16)] = 1
    w |= {"l0.mix.q": X.to_bf16(q), "l0.mix.dkv": X.to_bf16(dkv), "l0.mix.uk": X.to_bf16(uk)}
    want = F.forward(c, w, toks)
    apart = X.error(F.forward(c, w, without)[-1:], want[-1:])
    assert apart > 0.25, apart  # the key is what the last row is about
    gpu.say(f"fuvolix far key {place} {dtype}")
    m = load(tmp_path, c, w, context=333, dtype=dtype)
    for sizes in ([333], [300, 32, 1], [100, 2, 64]):
        e = X.error(in_portions(m, toks, sizes), want)
        assert e < TOL[dtype], (sizes, e)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("layer", [X.lightning(heads=2, decay=[1.0, 1.0]), X.mlstm(heads=2)], ids=["lightning", "mlstm"])
def test_one_far_position_in_a_state(tmp_path, layer, dtype):
    """A position whose key and value are far larger than the others', in a state that hardly forgets: every later row
    carries it, over chunk edges and into decoding."""
    c = X.config([layer], width=64, vocab=50, groups=1, taps=1)
    # only token 45 has the first feature; keys, values and the input gate grow with it
    w = changed(X.weights(c, 6), canon1=off, dwa=lambda t: np.array([0.0, 1.0]), embed=lambda t: t * (np.arange(64) > 0) + 6 * np.eye(50, 64, -45))
    loud = lambda t: t + 4 * (np.arange(64) == 0)
    w = changed(w, k=loud, v=loud, **({"f__b": lambda t: t * 0 + 8, "f": off, "i__b": lambda t: t * 0 - 2, "i": lambda t: loud(t * 0)} if layer["type"] == "mlstm" else {}))
    toks = X.tokens(c, 200, 3) % 40
    for place in (0, 62, 63, 64, 130):
        one = toks.copy()
        one[place] = 45
        want = F.forward(c, w, one)
        apart = X.error(F.forward(c, w, toks)[-1:], want[-1:])
        assert apart > 0.25, apart  # it is still what the last row is about
        gpu.say(f"fuvolix far position {layer['type']} {place} {dtype}")
        m = load(tmp_path, c, w, context=200, dtype=dtype)
        for sizes in ([200], [64, 1], [190, 1, 2]):
            assert X.error(in_portions(m, one, sizes), want) < TOL[dtype], (place, sizes)


SIZES = {
    "odd": X.config([X.latent(heads=5, dim=10, rot_dim=6, vdim=7, kv_rank=21, ff=33), X.mlstm(heads=5, dim=9, vdim=7), X.lightning(heads=7, dim=5, vdim=11)], width=75,
                    vocab=101, groups=5, taps=2, eps=1e-3),
    "one_of_each": X.config([X.latent(heads=1, dim=1, rot_dim=2, vdim=1, kv_rank=1, ff=1), X.mlstm(heads=1, dim=1, vdim=1), X.lightning(heads=1, dim=1, vdim=1, decay=[0.9])],
                            width=32, vocab=40, groups=1, taps=1),
    "many_heads": X.config([X.latent(heads=33, dim=8, rot_dim=8, vdim=8, kv_rank=72), X.mlstm(heads=19, dim=8, vdim=8), X.lightning(heads=17, dim=8, vdim=8)], width=160, groups=4),
    "wide_heads": X.config([X.latent(heads=2, dim=128, rot_dim=64, vdim=128, kv_rank=512, ff=512), X.mlstm(heads=2, dim=128, vdim=192), X.lightning(heads=2, dim=256, vdim=136)],
                           width=256, groups=4),
    "wider_heads": X.config([X.latent(heads=2, dim=192, rot_dim=32, vdim=160, kv_rank=600), X.mlstm(heads=1, dim=256, vdim=64), X.lightning(heads=2, dim=64, vdim=256)], width=192),
    "past_the_prompt_kernel": X.config([X.latent(heads=2, dim=300, rot_dim=10, vdim=288, kv_rank=96)], width=96),
    "latents": X.config([X.latent(heads=35, dim=16, rot_dim=104, vdim=16, kv_rank=504), X.latent(heads=4, dim=8, rot_dim=40, vdim=40, kv_rank=200),
                         X.latent(heads=4, dim=8, rot_dim=6, vdim=24, kv_rank=124)], width=96),
    "eight_rows_wide": X.config([X.latent(heads=2, dim=96, rot_dim=24, vdim=72, kv_rank=88), X.mlstm(heads=3, dim=24, vdim=104)], width=2080, groups=13),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", SIZES)
def test_other_sizes(tmp_path, name, dtype):
    c = SIZES[name]
    w = X.weights(c, 7)
    toks = X.tokens(c, 140, 7)
    want = F.forward(c, w, toks)
    gpu.say(f"fuvolix sizes {name} {dtype}")
    m = load(tmp_path, c, w, context=140, dtype=dtype)
    for sizes in ([140], [67, 2, 40, 1]):
        e = X.error(in_portions(m, toks, sizes), want)
        print(name, dtype, sizes, e)
        assert e < TOL[dtype], (sizes, e)


def test_gates_and_states_far_from_one(tmp_path):
    """Gates driven to their cap in both directions, and a state that decays to nothing and starts anew. A state of one
    key only gives o = v sign(k . q): the few rows where k . q is within its rounding of zero are not looked at."""
    c = X.config([X.mlstm(gate_cap=15.0)])
    w = changed(X.weights(c, 8), i=lambda t: t * 12, f=lambda t: t * 12)
    toks = X.tokens(c, 150, 8)
    want = F.forward(c, w, toks)
    gpu.say("fuvolix strong gates")
    for dtype in DTYPES:
        m = load(tmp_path, c, w, dtype=dtype)
        for sizes in ([150], [1], [65, 20]):
            e = X.error(in_portions(m, toks, sizes), want, quantile=0.95)
            print(dtype, sizes, e)
            assert e < TOL[dtype]


def test_greedy_generation(mixed):
    """The greedy loop (a recorded step; the same launches one by one; calls with the position from the host) in float32
    against the plain forward's choices, far into decoding. Where the two best logits are close, either may be chosen."""
    c, w, toks, _, folder = mixed
    lib = gpu.lib()
    m = registry.load(folder, context=256, dtype="float32")
    prompt, n = toks[:70], 120
    gpu.say("fuvolix greedy")
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
        lg = F.forward(c, w, np.concatenate([prompt, out]))[69:-1]
        chosen = lg[np.arange(n), out]
        assert np.all(lg.max(1) - chosen < 1e-3 * lg.std())
    # generation goes on from what the sequence holds
    more = m.logits_at([int(replayed[0, -1])], [0])
    assert X.error(more, F.forward(c, w, np.concatenate([prompt, replayed[0]]))[-1:]) < TOL["float32"]


@pytest.mark.parametrize("dtype", DTYPES)
def test_generation_of_several_sequences(mixed, dtype):
    """Each of the sequences chooses as it does alone (bfloat16: as long as no two logits are closer than its rounding)."""
    c, w, _, _, folder = mixed
    gpu.say(f"fuvolix greedy batch {dtype}")
    prompts = X.tokens(c, 40, 11, batch=10)  # more rows than one product of few rows takes
    m = registry.load(folder, context=96, batch=10, dtype=dtype)
    out, _ = m.generate(prompts, 24)
    for b in (0, 4, 9):
        lg = F.forward(c, w, np.concatenate([prompts[b], out[b]]))[39:-1]
        behind = lg.max(1) - lg[np.arange(24), out[b]]
        assert np.all(behind < (1e-3 if dtype == "float32" else 0.25) * lg.std()), behind.max() / lg.std()


def test_errors_before_anything_runs(tmp_path, mixed):
    c, w, toks, _, folder = mixed
    gpu.say("fuvolix errors")
    m = registry.load(folder, context=20, dtype="float32")
    with pytest.raises(capi.Mi355xError) as e:
        m.logits(toks[:21])
    assert e.value.status == capi.ERR_SHAPE
    with pytest.raises(capi.Mi355xError) as e:
        m.logits([0, c["vocab"]])
    assert e.value.status == capi.ERR_INDEX
    with pytest.raises(capi.Mi355xError) as e:
        m.logits_at(toks[:5], [5])
    assert e.value.status == capi.ERR_INDEX
    assert m.cache_len == 0
    part = dict(w)
    del part["l1.mix.uk"]
    with pytest.raises(capi.Mi355xError, match="l1.mix.uk"):
        load(tmp_path, c, part)
    with pytest.raises(capi.Mi355xError, match="elements"):
        load(tmp_path, c, w | {"l2.mix.i": w["l2.mix.i"][:1]})
    with pytest.raises(capi.Mi355xError, match="unknown tensor"):
        load(tmp_path, c, w | {"l0.mix.z": w["l2.mix.i"]})


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay(tmp_path, mixed, dtype):
    """bin/trace_run: requests one after the other, cut into steps; its logits are the handle's."""
    c, w, toks, want, folder = mixed
    steps = [dict(step=0, entries=[dict(id="a", tokens=toks[:50].tolist(), want=[0, 49])], end=[]),
             dict(step=1, entries=[dict(id="a", tokens=toks[50:52].tolist(), want=[])], end=[]),
             dict(step=2, entries=[dict(id="a", tokens=toks[52:53].tolist(), want=[0])], end=["a"]),
             dict(step=3, entries=[dict(id="b", tokens=toks[:12].tolist(), want=[11, 3])], end=["b"])]
    gpu.say(f"fuvolix trace {dtype}")
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
