"""What of the Fuvolix design can be held without a GPU: the plain forward's mechanisms against other formulations of
them, and the reading of a model's folder."""
import json
import os
import re

import numpy as np
import pytest

from mimir_amd import build, capi, registry, stack
from mimir_amd.safetensors import SafetensorsError, SafetensorsFile
from oracle import fuvolix as F
from tests import fuvolix as X

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def _rng():
    return np.random.default_rng(0)


def test_group_norm_is_each_part_over_its_own_root_mean_square():
    x, w = _rng().normal(size=(4, 12)) * 10.0 ** np.arange(12), _rng().normal(size=12)
    y = F.group_norm(x, w, 3, 1e-6)
    for g in range(3):
        part = x[:, 4 * g:4 * g + 4]
        assert np.allclose(y[:, 4 * g:4 * g + 4], part / np.sqrt((part ** 2).sum(1, keepdims=True) / 4 + 1e-6) * w[4 * g:4 * g + 4])
    assert not np.allclose(y, F.group_norm(x, w, 1, 1e-6))


def test_causal_conv_is_a_convolution():
    h, w = _rng().normal(size=(20, 3)), _rng().normal(size=(3, 4))
    for c in range(3):
        assert np.allclose(F.causal_conv(h, w)[:, c], np.convolve(h[:, c], w[c, ::-1])[:20])
    assert np.allclose(F.causal_conv(h, w[:, :1]), h * w[:, 0])


def test_rotation_turns_pairs_and_scores_see_distances():
    x = _rng().normal(size=(9, 6))
    y = F.rotate(x, np.arange(9), 100.0)
    assert np.allclose(y[0], x[0]) and np.allclose((y ** 2).reshape(9, 3, 2).sum(2), (x ** 2).reshape(9, 3, 2).sum(2))
    a, b = x[:1], x[1:2]
    score = lambda i, j: (F.rotate(a, np.array([i]), 100.0) @ F.rotate(b, np.array([j]), 100.0).T)[0, 0]
    assert np.isclose(score(7, 3), score(104, 100)) and not np.isclose(score(7, 3), score(7, 4))
    assert np.isclose(y[5, 0], x[5, 0] * np.cos(5) - x[5, 1] * np.sin(5))  # the first pair turns by one radian a position


def test_latent_attention_without_forming_keys():
    """Queries taken to the latents' space give the scores of formed keys; and no row sees a later one."""
    c = X.config([X.latent()])
    t = F.sub(X.weights(c, 1), "l0.mix.")
    mx, h = c["layers"][0]["mixer"], _rng().normal(size=(30, 96))
    y = F.latent_attention(h, t, mx, 1e-5)
    H, d, r, rank = mx["heads"], mx["dim"], mx["rot_dim"], mx["kv_rank"]
    q, low = (h @ t["q"].T).reshape(30, H, d + r), h @ t["dkv"].T
    lat = F.rms(low[:, :rank], 1e-5) * t["dkv.norm"]
    out = []
    for a in range(H):
        qa = q[:, a, :d] @ t["uk"].reshape(H, d, rank)[a]
        s = (qa @ lat.T + F.rotate(q[:, a, d:], np.arange(30), mx["rot"]["base"]) @ F.rotate(low[:, rank:], np.arange(30), mx["rot"]["base"]).T) * mx["scale"]
        p = np.exp(s) * np.tri(30)
        out.append(p / p.sum(1, keepdims=True) @ lat @ t["uv"].reshape(H, mx["vdim"], rank)[a].T)
    assert np.allclose(y, np.concatenate(out, 1) @ t["o"].T)
    h2 = h.copy()
    h2[20:] += 1
    assert np.allclose(F.latent_attention(h2, t, mx, 1e-5)[:20], y[:20])


def test_mlstm_scan_is_the_unstabilized_recurrence():
    """With gates of moderate size: the sums weighted by exp of log gates, over max(|n . q|, 1) in the stabilized scale."""
    rng = _rng()
    n, H, d, e = 25, 2, 4, 3
    q, k, v = rng.normal(size=(n, H, d)), rng.normal(size=(n, H, d)), rng.normal(size=(n, H, e))
    i, f = rng.normal(size=(n, H)), F.logsigmoid(rng.normal(size=(n, H)) + 1)
    got = F.mlstm_scan(q, k, v, i, f)
    for a in range(H):
        m = 0.0
        for t in range(n):
            m = max(f[t, a] + m, i[t, a])
            w = np.array([np.exp(f[s + 1:t + 1, a].sum() + i[s, a]) for s in range(t + 1)])
            dots = w * (k[:t + 1, a] @ q[t, a])
            want = np.exp(-m) * (dots @ v[:t + 1, a]) / (max(abs(np.exp(-m) * dots.sum()), np.exp(-m)) + 1e-6)
            assert np.allclose(got[t, a], want)


def test_lightning_scan_is_a_decayed_sum():
    rng = _rng()
    q, k, v = rng.normal(size=(20, 2, 4)), rng.normal(size=(20, 2, 4)), rng.normal(size=(20, 2, 3))
    got = F.lightning_scan(q, k, v, np.array([0.5, 1.0]))
    for a, dec in enumerate((0.5, 1.0)):
        w = np.tril(dec ** np.maximum(np.arange(20)[:, None] - np.arange(20), 0))
        assert np.allclose(got[:, a], (w * (q[:, a] @ k[:, a].T)) @ v[:, a])


def test_depth_average_and_residual_order():
    """Two layers whose mixers give nothing: what is left is the average of the embedding output and itself."""
    c = X.config([X.lightning(), X.lightning(ff=8)])
    w = {k: (v * 0 if k.endswith((".o", ".down")) else v) for k, v in X.weights(c).items()}
    streams = []
    logits = F.forward(c, w, [3, 4], streams)
    x = F.group_norm(w["embed"][[3, 4]].astype(np.float64), w["embed.norm"], 3, 1e-5)
    a, b = w["l0.dwa"].astype(np.float64), w["l1.dwa"].astype(np.float64)
    y = a.sum() * x
    z = (b[0] + b[1] + b[2] * a.sum()) * x
    # what a layer adds to is the averaged residual; what later averages take of it is its result before its own average
    assert np.allclose(streams[0], y) and np.allclose(streams[1], z)
    assert np.allclose(logits, F.group_norm(z, w["final.norm"], 3, 1e-5) @ w["embed"].T)


def test_config_reader():
    c = X.config([X.latent(ff=40), X.mlstm(gate_cap=7.0), X.lightning(decay=[0.25, 0.5, 1.0])], taps=5, groups=2, eps=2e-4)
    s, layers = stack.fuvolix_config(c, context=77, batch=3, dtype="float32")
    assert (s.width, s.vocab, s.layers, s.context, s.batch, s.taps, s.norm_groups, s.dtype, s.eps) == (96, 130, 3, 77, 3, 5, 2, capi.F32, 2e-4)
    a, b, d = layers
    assert (a.mixer, a.heads, a.dim, a.vdim, a.rot_dim, a.kv_rank, a.ff, a.rot_base, a.scale) == (capi.MIXER_LATENT, 3, 16, 24, 8, 40, 40, 500.0, 24 ** -0.5)
    assert (b.mixer, b.gate_cap, b.ff) == (capi.MIXER_MLSTM, 7.0, 0)
    assert d.mixer == capi.MIXER_LIGHTNING and list(d.decay[:3]) == [0.25, 0.5, 1.0]
    for edit in (dict(type="window"), dict(mlp=dict(kind="gated", ff=4))):
        with pytest.raises(ValueError, match="layer 0"):
            stack.fuvolix_config(X.config([X.mlstm() | edit]), 10)
    with pytest.raises(ValueError, match="decays"):
        stack.fuvolix_config(X.config([X.lightning(decay=[0.5])]), 10)


def test_registry_names_what_a_path_holds(tmp_path, golden_dir):
    c = X.config([X.mlstm()])
    assert registry.architecture(X.write(tmp_path, c, X.weights(c))) == "Fuvolix"
    assert registry.architecture(os.path.join(golden_dir, "spm.mim")) == "llama"
    assert registry.architecture(os.path.join(golden_dir, "qwen2-exact.mim")) == "qwen2"
    (tmp_path / "config.json").write_text(json.dumps(dict(c, architecture="Other")))
    with pytest.raises(ValueError, match="Other"):
        registry.architecture(str(tmp_path))


def test_safetensors(tmp_path):
    c = X.config([X.latent()])
    w = X.weights(c)
    f = SafetensorsFile(os.path.join(X.write(tmp_path, c, w), "model.safetensors"))
    assert set(f.tensors) == set(w)
    for name, (dt, data) in f.tensors.items():
        assert dt == "BF16" and data.shape == w[name].shape
        assert np.array_equal((data.astype(np.uint32) << 16).view(np.float32), w[name])
    path = tmp_path / "model.safetensors"
    raw = path.read_bytes()
    path.write_bytes(raw[:-2])
    with pytest.raises(SafetensorsError, match="bytes"):
        SafetensorsFile(str(path))
    path.write_bytes(raw[:20])
    with pytest.raises(SafetensorsError, match="cut short"):
        SafetensorsFile(str(path))


def test_parts_of_the_library_are_sources_that_exist():
    whole = set(build.sources())
    for part in build.PARTS:
        assert set(build.sources(part)) < whole
    for arch, (_, part) in registry.ARCHITECTURES.items():
        assert part is None or part in build.PARTS, arch


def test_configuration_errors_come_before_a_device_is_touched():
    lib = capi.load()
    import ctypes as C
    h = C.c_void_p()

    def create(c, **edit):
        s, layers = stack.fuvolix_config(c, 16)
        for k, v in edit.items():
            setattr(s if hasattr(s, k) else layers[0], k, v)
        st = lib.mi355x_stack_create(C.byref(s), (capi.StackLayer * len(layers))(*layers), C.byref(h))
        if st == capi.OK:
            lib.mi355x_model_destroy(h)
        return st

    ok = X.config([X.latent(ff=8), X.mlstm(), X.lightning()])
    assert create(ok) == capi.OK
    for edit in (dict(norm_groups=7), dict(taps=-1), dict(width=0), dict(context=0), dict(eps=0.0), dict(rot_dim=7), dict(kv_rank=0), dict(heads=0), dict(mixer=9)):
        assert create(ok, **edit) == capi.ERR_SHAPE, edit
    assert create(ok, dtype=capi.F16) == capi.ERR_DTYPE
    assert create(X.config([X.mlstm(dim=257)])) == capi.ERR_SHAPE


def test_part_exports_the_entry_points_its_models_call():
    """The handle's entry points and the stack's live in the part's sources."""
    text = "".join(open(f).read() for f in build.sources("stack"))
    for name in capi.SYMBOLS:
        if name.startswith(("mi355x_model_", "mi355x_stack_")) or name in ("mi355x_init", "mi355x_last_error", "mi355x_sync"):
            assert re.search(rf"\b{name}\(", text), name
