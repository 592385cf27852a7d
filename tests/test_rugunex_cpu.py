"""Rugunex without a GPU: configuration and registry errors, rotary tables of the engine (host code) against the oracle, and identities of the
oracle itself."""
import ctypes as C
import json

import numpy as np
import pytest

import mlx_audio_swift_amd as mas
from mlx_audio_swift_amd import _lib, registry
from oracle import rugunex as orc
from rugunex_util import config, mixer


@pytest.mark.parametrize("dims,base,scaling", [
    (10, 10000.0, None), (2, 500.0, None), (64, 1e6, None),
    (64, 1e4, dict(factor=4.0, original=2048, fast=32.0, slow=1.0)),
    (48, 5e5, dict(factor=40.0, original=4096, fast=16.0, slow=2.0)),
    (8, 100.0, dict(factor=2.5, original=64, fast=32.0, slow=1.0)),          # the ramp's start is clamped to pair 0
    (6, 10.0, dict(factor=16.0, original=1 << 20, fast=4.0, slow=0.5)),      # ... and its end to dims - 1
    (16, 1e4, dict(factor=3.0, original=512, fast=2.0, slow=2.0)),           # fast = slow
])
def test_rotary_tables(dims, base, scaling):
    n = 700
    cs, sn = np.zeros((n, dims // 2), np.float32), np.zeros((n, dims // 2), np.float32)
    s = scaling or dict(factor=1.0, original=1.0, fast=1.0, slow=1.0)
    assert _lib.lib().mis_debug_rotary_tables(dims, base, int(scaling is not None), s["factor"], s["original"], s["fast"], s["slow"], n,
                                              cs.ctypes.data, sn.ctypes.data) == 0
    f, mag = orc.rotary_frequencies(dims, base, scaling), orc.rotary_magnitude(scaling)
    ang = np.arange(n)[:, None] * f[None, :]
    assert np.abs(cs - mag * np.cos(ang)).max() < 2e-7 * mag * 2
    assert np.abs(sn - mag * np.sin(ang)).max() < 2e-7 * mag * 2
    assert scaling is None or mag > 1.0


def test_rotation_is_interleaved_and_relative():
    g = np.random.default_rng(0)
    f = orc.rotary_frequencies(8, 1e4)
    x, y = g.standard_normal((2, 1, 12))
    a = orc.rotate_interleaved(x, [3], f)
    assert np.allclose(a[0, 8:], x[0, 8:])                                     # dimensions past the rotated ones pass through
    u, v = x[0, 2], x[0, 3]
    assert np.allclose(a[0, 2:4], [u * np.cos(3 * f[1]) - v * np.sin(3 * f[1]), v * np.cos(3 * f[1]) + u * np.sin(3 * f[1])])

    def dot(i, j):
        return float((orc.rotate_interleaved(x, [i], f) @ orc.rotate_interleaved(y, [j], f).T)[0, 0])
    assert abs(dot(5, 2) - dot(105, 102)) < 1e-9 and abs(dot(5, 2) - dot(5, 3)) > 1e-3


def test_window_and_softmax():
    m = orc.window_mask(9, 4)
    assert m[8].tolist() == [False] * 5 + [True] * 4 and m[1].tolist() == [True, True] + [False] * 7
    assert orc.window_mask(5, None)[4].all()
    w = orc.masked_softmax(np.random.default_rng(1).standard_normal((9, 9)) * 30, m)
    assert np.allclose(w.sum(1), 1) and (w[~m] == 0).all()


def test_absorbed_form_is_the_expanded_form():
    """q . (W_uk c) = (W_uk^T q) . c and W_uv (sum p c) = sum p (W_uv c): what the decode kernels rely on."""
    cfg = config(layers=[dict(mixer=mixer(window=5))])
    mx, W = cfg["layers"][0]["mixer"], orc.random_weights(cfg, 3)
    w = {k[4:]: v for k, v in orc.layer_weights(W, 0).items() if k.startswith("mix.")}
    h = np.random.default_rng(4).standard_normal((11, cfg["width"]))
    ref = orc.latent_attention(h, mx, w, 1e-6)
    H, n, r, v, R = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
    q = (h @ w["q"].T.astype(np.float64)).reshape(11, H, n + r)
    c, k_r = orc.latent(h, w["dkv"], w["dkv.norm"], R, 1e-6)
    f, mag = orc.rotary_frequencies(mx["rot"]["dims"], mx["rot"]["base"], mx["rot"].get("scaling")), orc.rotary_magnitude(mx["rot"].get("scaling"))
    q_r, k_r = orc.rotate_interleaved(q[:, :, n:], np.arange(11), f, mag), orc.rotate_interleaved(k_r, np.arange(11), f, mag)
    uk, uv = w["uk"].reshape(H, n, R).astype(np.float64), w["uv"].reshape(H, v, R).astype(np.float64)
    out = np.zeros((11, H, v))
    for a in range(H):
        s = ((q[:, a, :n] @ uk[a]) @ c.T + q_r[:, a] @ k_r.T) * mx["scale"]
        out[:, a] = (orc.masked_softmax(s, orc.window_mask(11, 5)) @ c) @ uv[a].T
    assert np.allclose(out.reshape(11, -1) @ w["o"].T.astype(np.float64), ref)


def test_window_reach_of_the_oracle():
    """A token changes logits up to (layers x (window - 1)) places behind it and nothing before it."""
    cfg = config(layers=[dict(mixer=mixer(window=3))])
    W = orc.random_weights(cfg, 5)
    t = list(range(12))
    a, b = orc.forward(cfg, W, t), orc.forward(cfg, W, t[:4] + [77] + t[5:])
    changed = np.abs(a - b).max(1) > 1e-9
    assert changed.tolist() == [False] * 4 + [True] * 3 + [False] * 5


def _create(cfg, compute=0):
    h = C.c_void_p()
    st = _lib.lib().mis_lm_create(json.dumps(cfg).encode(), compute, 0, C.byref(h))
    if st == 0:
        _lib.lib().mis_tts_destroy(h)
    return st, _lib.last_error()


def test_configuration_errors_are_found_before_the_device():
    ok = config()
    assert _create({**ok, "architecture": "Other"})[0] == 3
    for key in ("width", "vocab", "layers", "norm"):
        st, msg = _create({k: v for k, v in ok.items() if k != key})
        assert st == 3 and key in msg
    bad = config()
    bad["layers"][0]["type"] = "recurrent"
    assert _create(bad)[0] == 3
    for key in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "scale", "rot"):
        bad = config()
        del bad["layers"][0]["mixer"][key]
        st, msg = _create(bad)
        assert st == 3 and key in msg
    bad = config()
    bad["layers"][0]["mixer"]["rot"]["dims"] = bad["layers"][0]["mixer"]["rot_dim"] + 2
    assert _create(bad)[0] == 3
    bad = config(layers=[dict(mixer=mixer()), dict(mixer=mixer(), weights_of=2)])
    assert _create(bad)[0] == 3
    bad = config(layers=[dict(mixer=mixer()), dict(mixer=mixer(heads=7), weights_of=0)])
    assert _create(bad)[0] == 3
    bad = config(layers=[dict(mixer=mixer(), weights_of=1), dict(mixer=mixer(), weights_of=0)])
    assert _create(bad)[0] == 3
    assert _create(ok, compute=7)[0] == 3
    if _lib.lib().mis_device_count() == 0:
        assert _create(ok)[0] == 7                                              # device: no CPU fallback


def test_registry(tmp_path):
    assert registry.model_class({"architecture": "Rugunex"}) is mas.BlockLanguageModel
    assert registry.model_class({"model_type": "llama"}) is mas.LlamaTTSModel and registry.model_class({}) is mas.LlamaTTSModel
    for bad in ({"architecture": "Nothing"}, {"model_type": "mamba"}):
        with pytest.raises(mas.AudioGenerationError) as e:
            registry.model_class(bad)
        assert e.value.case == "invalidInput"
    with pytest.raises(mas.AudioGenerationError):
        mas.BlockModelConfiguration.from_dict({"architecture": "Rugunex", "width": 8})
    (tmp_path / "config.json").write_text(json.dumps({"model_type": "llama"}))
    with pytest.raises(mas.AudioGenerationError) as e:                          # the Llama chain has no 32-bit mode
        registry.load_model(str(tmp_path), compute="float32")
    assert e.value.case == "invalidInput"
