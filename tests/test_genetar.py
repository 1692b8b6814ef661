"""What of the Genetar design can be held without a GPU: the plain forward's mechanisms against other formulations of
them, that a mistake in one shows, and the reading of a model's folder."""
import ctypes as C
import json
import os

import numpy as np
import pytest

from mimir_amd import capi, registry, stack
from mimir_amd.safetensors import SafetensorsFile
from oracle import genetar as G
from tests import genetar as X


def _rng():
    return np.random.default_rng(0)


def test_pairs_of_tokens():
    table, pairs = _rng().normal(size=(9, 4)), _rng().normal(size=(6, 4))
    x = G.embed_pairs([3, 8, 8, 0], table, pairs, 7, 2)
    assert np.allclose(x[0], table[3] + pairs[5])  # nothing before it: the last row
    assert np.allclose(x[1], table[8] + pairs[(3 * 7 + 8 * 2) % 5])
    assert np.allclose(x[2], table[8] + pairs[(8 * 7 + 8 * 2) % 5])
    assert np.allclose(x[3], table[0] + pairs[(8 * 7) % 5])


def test_frequencies_are_kept_stretched_and_between():
    rot = dict(base=1000.0, dims=24, scaling=dict(factor=5.0, low=1.0, high=4.0, original=200))
    plain, f = G.frequencies(dict(rot, scaling=None)), G.frequencies(rot)
    assert np.allclose(plain, 1000.0 ** (-np.arange(12) / 12))
    turns = 200 * plain / (2 * np.pi)  # of the original length
    assert (turns > 4).any() and (turns < 1).any() and ((turns >= 1) & (turns <= 4)).any()
    assert np.allclose(f[turns > 4], plain[turns > 4]) and np.allclose(f[turns < 1], plain[turns < 1] / 5)
    t = turns[(turns >= 1) & (turns <= 4)]
    assert np.allclose(f[(turns >= 1) & (turns <= 4)] / plain[(turns >= 1) & (turns <= 4)], 1 / 5 + (1 - 1 / 5) * (t - 1) / 3)
    assert np.all(np.diff(f) < 0)


def test_rotation_turns_halves_and_leaves_the_rest():
    rot = dict(base=50.0, dims=6)
    x = _rng().normal(size=(9, 2, 10))
    y = G.rotate_halves(x, np.arange(9), rot)
    assert np.allclose(y[0], x[0]) and np.array_equal(y[..., 6:], x[..., 6:])
    z = (x[..., :3] + 1j * x[..., 3:6]) * np.exp(1j * np.arange(9)[:, None, None] * 50.0 ** (-np.arange(3) / 3))
    assert np.allclose(y[..., :3], z.real) and np.allclose(y[..., 3:6], z.imag)


def test_attention_of_groups_with_a_cap():
    rng = _rng()
    q, k, v = rng.normal(size=(12, 6, 5)) * 3, rng.normal(size=(12, 2, 5)), rng.normal(size=(12, 2, 4))
    out = G.softmax_attend(q, k, v, 0.8, 2.0)
    for i in (0, 5, 11):
        for h in range(6):
            s = 2.0 * np.tanh(k[:i + 1, h // 3] @ q[i, h] * 0.8 / 2.0)
            w = np.exp(s) / np.exp(s).sum()
            assert np.allclose(out[i, h], w @ v[:i + 1, h // 3])
    assert np.allclose(G.softmax_attend(q, k, v, 0.8, None), G.softmax_attend(q, k, v, 0.8, 1e7), atol=1e-9)


def test_values_of_the_first_mixing_layer_are_what_others_mix_in():
    mx = X.unit(v_mix=True)["mixer"]
    c = X.config([X.unit(), X.unit()])
    t = G.sub(X.weights(c, 1), "l1.mix.")
    h = _rng().normal(size=(7, 80))
    own = (h @ t["v"].T).reshape(7, 2, 16)
    a, first = G.attention(h, t, mx, 1e-5, None, True, None, False)
    assert np.allclose(first, own)
    other = _rng().normal(size=own.shape)
    b, kept = G.attention(h, t, mx, 1e-5, other, True, None, False)
    assert kept is other and not np.allclose(a, b)
    # a value of the mix goes through linearly
    lam = float(t["vmix"])
    c0, _ = G.attention(h, dict(t, v=t["v"] * 0), mx, 1e-5, other, True, None, False)
    assert np.allclose(b, (1 - lam) * a + c0)
    _, none = G.attention(h, t, dict(mx, v_mix=False), 1e-5, None, True, None, False)
    assert none is None


def test_sublayers_read_one_norm_and_have_a_scale_each():
    c = X.config([X.rotary(ff=24)])
    w = {k: v.astype(np.float64) for k, v in X.weights(c, 2).items()}
    toks, streams = [5, 1, 1], []
    G.forward(c, w, toks, streams)
    x = G.embed_pairs(toks, w["embed"], w["bigram"], 11, 5)
    h = G.unit_rms(x, 1e-5) * w["l0.norm1"]
    o, _ = G.attention(h, G.sub(w, "l0.mix."), c["layers"][0]["mixer"], 1e-5, None, False, c["layers"][0]["mixer"]["rot"], True)
    m = (G.silu(h @ w["l0.mlp.gate"].T) * (h @ w["l0.mlp.up"].T)) @ w["l0.mlp.down"].T
    assert np.allclose(streams[0], x + o * w["l0.ls1"] + m * w["l0.ls2"])


@pytest.mark.parametrize("mistake", ["pair", "first_pair", "unit", "cap", "scaling", "halves", "gate", "mix", "mix_all", "scale"])
def test_a_mistake_in_one_mechanism_shows(mistake, monkeypatch):
    """Each of these, planted in the plain forward, moves the logits of the tests' models by far more than their tolerances."""
    c = X.config([X.unit(ff=40), X.rotary(), X.unit()])
    w = X.weights(c, 3)
    toks = X.tokens(c, 60)
    want = G.forward(c, w, toks)
    if mistake == "pair":
        c["embedding"]["bigram"]["mul_prev"], c["embedding"]["bigram"]["mul_cur"] = 5, 11
    elif mistake == "first_pair":
        w["bigram"][-1] = w["bigram"][0]
    elif mistake == "unit":
        monkeypatch.setattr(G, "unit_rms", lambda x, eps, f=G.unit_rms: x if x.ndim == 3 else f(x, eps))
    elif mistake == "cap":
        monkeypatch.setattr(G, "soft_cap", lambda s, cap: np.clip(s, -1, 1))
    elif mistake == "scaling":
        c["layers"][1]["mixer"]["rot"]["scaling"] = None
        monkeypatch.setattr(G, "frequencies", lambda rot: rot["base"] ** (-2.0 * np.arange(rot["dims"] // 2)))
    elif mistake == "halves":
        turn = G.rotate_halves
        swap = [0, 5, 1, 6, 2, 7, 3, 8, 4, 9] + list(range(10, 24))
        monkeypatch.setattr(G, "rotate_halves", lambda x, p, rot: turn(x[..., np.argsort(swap)], p, rot)[..., swap])
    elif mistake == "gate":
        monkeypatch.setattr(G, "sigmoid", lambda z: np.ones_like(z) if z.shape[-1] == 6 else 1 / (1 + np.exp(-z)))
    elif mistake == "mix":
        w["l2.mix.vmix"] = w["l2.mix.vmix"] * 0
    elif mistake == "mix_all":
        c["layers"][0]["mixer"]["v_mix"] = False  # the second becomes the first
    else:
        w["l0.ls1"], w["l0.ls2"] = w["l0.ls2"], w["l0.ls1"]
    got = G.forward(c, w, toks)
    rows = slice(0, 1) if mistake == "first_pair" else slice(None)
    assert X.error(got[rows], want[rows]) > 0.1


def test_config_reader():
    c = X.config([X.unit(ff=40, softcap=9.0), X.rotary(heads=4, kv_heads=4, dim=32, vdim=8, scale=0.3, v_mix=False, rot=20, base=77.0)], logit_scale=0.125, eps=3e-6,
                 buckets=55, mul_prev=301, mul_cur=2)
    s, layers = stack.genetar_config(c, context=77, batch=3, dtype="float32")
    assert (s.width, s.vocab, s.layers, s.context, s.batch, s.taps, s.norm_groups, s.dtype, s.eps) == (80, 130, 2, 77, 3, 0, 1, capi.F32, 3e-6)
    assert (s.pair_buckets, s.pair_mul_prev, s.pair_mul_cur, s.logit_scale) == (55, 301, 2, 0.125)
    assert s.flags == capi.STACK_PARALLEL | capi.STACK_LAYER_SCALE | capi.STACK_OUTPUT_MATRIX
    a, b = layers
    assert (a.mixer, a.heads, a.kv_heads, a.dim, a.vdim, a.ff, a.mlp, a.softcap, a.unit_qk, a.value_mix, a.head_gate, a.rot_dim) == \
        (capi.MIXER_ATTENTION, 6, 2, 24, 16, 40, capi.MLP_SWIGLU, 9.0, 1, 1, 0, 0)
    assert (b.heads, b.kv_heads, b.dim, b.vdim, b.ff, b.scale, b.unit_qk, b.value_mix, b.head_gate) == (4, 4, 32, 8, 0, 0.3, 0, 0, 1)
    assert (b.rot_dim, b.rot_base, b.rot_factor, b.rot_low, b.rot_high, b.rot_original) == (20, 77.0, 3.0, 1.5, 6.0, 64.0)
    for edit in (dict(type="latent_attention"), dict(mlp=dict(kind="experts", ff=4))):
        with pytest.raises(ValueError, match="layer 0"):
            stack.genetar_config(X.config([X.unit() | edit]), 10)


def test_registry_and_folder(tmp_path):
    c = X.config([X.unit(), X.rotary()])
    w = X.weights(c)
    folder = X.write(tmp_path, c, w)
    assert registry.architecture(folder) == "Genetar"
    f = SafetensorsFile(os.path.join(folder, "model.safetensors"))
    assert f.tensors["l0.mix.vmix"][1].shape == () and set(f.tensors) == set(w)
    (tmp_path / "config.json").write_text(json.dumps(dict(c, architecture="Genetar2")))
    with pytest.raises(ValueError, match="Genetar2"):
        registry.architecture(folder)


def _create(c, **edit):
    lib, h = capi.load(), C.c_void_p()
    s, layers = stack.genetar_config(c, 16)
    for k, v in edit.items():
        setattr(s if hasattr(s, k) else layers[-1], k, v)
    st = lib.mi355x_stack_create(C.byref(s), (capi.StackLayer * len(layers))(*layers), C.byref(h))
    names = {}
    if st == capi.OK:
        name, n, k, i = C.create_string_buffer(64), C.c_int64(), C.c_int64(), 0
        while lib.mi355x_stack_tensor(h, i, name, 64, C.byref(n), C.byref(k)) == capi.OK:
            names[name.value.decode()] = n.value * k.value
            i += 1
        lib.mi355x_model_destroy(h)
    return st, names


def test_tensors_are_the_file_s():
    c = X.config([X.unit(ff=9), X.rotary(v_mix=False), X.rotary(ff=33)])
    st, names = _create(c)
    assert st == capi.OK
    want = {k: int(np.prod(v)) for k, v in X.shapes(c).items()}
    assert {k: names.get(k) for k in want} == want
    # what a file may hold beside them: a factor without a use
    assert set(names) - set(want) <= {"l1.ls2", "l1.mix.vmix"}


def test_configuration_errors_come_before_a_device_is_touched():
    ok = X.config([X.unit(ff=8), X.rotary()])
    assert _create(ok)[0] == capi.OK
    for edit in (dict(kv_heads=4), dict(kv_heads=0), dict(dim=1025), dict(vdim=1025), dict(rot_dim=9), dict(rot_dim=26), dict(softcap=-1.0), dict(taps=3),
                 dict(flags=capi.STACK_PARALLEL | capi.STACK_POST_NORMS), dict(pair_buckets=-1), dict(pair_mul_prev=-1), dict(mixer=capi.MIXER_MLSTM), dict(mlp=2),
                 dict(ff=4, mlp=capi.MLP_RELU2)):
        assert _create(ok, **edit)[0] == capi.ERR_SHAPE, edit
    # values that are mixed have one shape
    assert _create(X.config([X.unit(), X.rotary(vdim=8)]))[0] == capi.ERR_SHAPE
    assert _create(X.config([X.unit(), X.rotary(vdim=8, v_mix=False)]))[0] == capi.OK
