"""Vamunex without a GPU: configuration and registry errors, and identities of the oracle that the kernels rely on."""
import ctypes as C
import json

import numpy as np
import pytest

import mlx_audio_swift_amd as mas
from mlx_audio_swift_amd import _lib, registry
from oracle import vamunex as orc
from vamunex_util import config, left, lightning, odd, parallel, right


def test_rotation_pairs_halves_and_is_relative():
    g = np.random.default_rng(0)
    x, y = g.standard_normal((2, 1, 11))
    a = orc.rotate_half(x, [3], 8, 1e4)
    assert np.allclose(a[0, 8:], x[0, 8:])                                     # dimensions past the rotated ones pass through
    f = 1e4 ** (-2.0 * 1 / 8)
    u, v = x[0, 1], x[0, 5]
    assert np.allclose([a[0, 1], a[0, 5]], [u * np.cos(3 * f) - v * np.sin(3 * f), v * np.cos(3 * f) + u * np.sin(3 * f)])

    def dot(i, j):
        return float((orc.rotate_half(x, [i], 8, 1e4) @ orc.rotate_half(y, [j], 8, 1e4).T)[0, 0])
    assert abs(dot(5, 2) - dot(105, 102)) < 1e-9 and abs(dot(5, 2) - dot(5, 3)) > 1e-3
    cs, sn = np.zeros((40, 4), np.float32), np.zeros((40, 4), np.float32)      # the engine's tables
    assert _lib.lib().mis_debug_rotary_tables(8, 1e4, 0, 1.0, 1.0, 1.0, 1.0, 40, cs.ctypes.data, sn.ctypes.data) == 0
    b = orc.rotate_half(np.tile(x, (40, 1)), np.arange(40), 8, 1e4)
    assert np.allclose(x[0, :4] * cs - x[0, 4:8] * sn, b[:, :4], atol=1e-6) and np.allclose(x[0, 4:8] * cs + x[0, :4] * sn, b[:, 4:8], atol=1e-6)


def test_kept_window_and_sink():
    m = orc.kept_window_mask(12, 4, 2)
    assert m[11].tolist() == [True, True] + [False] * 6 + [True] * 4
    assert m[4].tolist() == [True] * 5 + [False] * 7 and m[1].tolist() == [True, True] + [False] * 10
    assert orc.kept_window_mask(6)[5].all()
    s = np.random.default_rng(1).standard_normal((12, 12)) * 20
    w = orc.sink_softmax(s, m, -1e9)
    assert np.allclose(w.sum(1), 1) and (w[~m] == 0).all()
    w = orc.sink_softmax(s, m, 3.0)
    z = np.exp(s[11][m[11]])
    assert np.allclose(w[11][m[11]], z / (z.sum() + np.exp(3.0)))


def test_decayed_state_in_chunks():
    """Within a chunk the state's part and the pair sums, between chunks one decayed update: what the prompt kernel relies on."""
    g = np.random.default_rng(2)
    T, D, E, C_ = 23, 5, 4, 7
    q, k, v = g.standard_normal((T, D)), g.standard_normal((T, D)), g.standard_normal((T, E))
    for dec in (0.0, 0.6, 1.0):
        ref = orc.decayed_outer_state(q, k, v, dec)
        S, out = np.zeros((D, E)), []
        for a in range(0, T, C_):
            qc, kc, vc = q[a:a + C_], k[a:a + C_], v[a:a + C_]
            n = len(qc)
            i = np.arange(n)
            pair = np.where(i[:, None] >= i[None, :], float(dec) ** np.maximum(i[:, None] - i[None, :], 0), 0.0)
            out.append(((qc @ kc.T) * pair) @ vc + (float(dec) ** (i + 1))[:, None] * (qc @ S))
            S = float(dec) ** n * S + (kc * (float(dec) ** (n - 1 - i))[:, None]).T @ vc
        assert np.allclose(np.concatenate(out), ref)


def test_gated_recurrence_in_chunks():
    """Local states from zero plus the carried state times the chunk's running product of decays."""
    g = np.random.default_rng(3)
    T, W = 20, 6
    u, lam = g.standard_normal((T, W)), g.standard_normal(W) - 2
    r, i = orc.sigmoid(g.standard_normal((T, W))), orc.sigmoid(g.standard_normal((T, W)))
    ref = orc.gated_recurrence(u, r, i, lam)
    la = -8.0 * r * np.log1p(np.exp(lam))
    S, out = np.zeros(W), []
    for a in range(0, T, 6):
        loc = orc.gated_recurrence(u[a:a + 6], r[a:a + 6], i[a:a + 6], lam)
        out.append(loc + np.exp(np.cumsum(la[a:a + 6], axis=0)) * S)
        S = out[-1][-1]
    assert np.allclose(np.concatenate(out), ref)


def test_norm_of_the_heads_commutes_with_the_output_product():
    cfg = config([lightning()])
    W = orc.random_weights(cfg, 5)
    o = np.random.default_rng(6).standard_normal((4, 90))
    w, g = W["l0.mix.norm"].astype(np.float64), np.random.default_rng(7).random((4, 90))
    r = 1.0 / np.sqrt(np.mean(o * o, axis=1, keepdims=True) + 1e-6)
    assert np.allclose(orc.linear(orc.rms(o, 1e-6) * w * g, W["l0.mix.o"]), r * orc.linear(o * w * g, W["l0.mix.o"]))


def test_convolution_and_blocks():
    x = np.random.default_rng(8).standard_normal((9, 3))
    taps = np.asarray([[0, 0, 1.0], [0, 1.0, 0], [1.0, 0, 0]])
    y = orc.causal_conv(x, taps, np.zeros(3))
    assert np.allclose(y[:, 0], x[:, 0]) and np.allclose(y[1:, 1], x[:-1, 1]) and np.allclose(y[2:, 2], x[:-2, 2]) and y[0, 1] == 0 and (y[:2, 2] == 0).all()
    w = np.zeros((2, 2, 2)); w[1, 0, 1] = 5.0
    assert np.allclose(orc.block_diagonal(np.ones((1, 4)), w, np.zeros((2, 2))), [[0, 0, 5, 0]])


def test_layer_order():
    assert orc.layer_order(odd()) == [0, 1, 2, 1, 2, 1, 2, 3]
    assert orc.layer_order(config([lightning(), lightning()])) == [0, 1]
    assert orc.layer_order(config([lightning(), lightning()], loop=(0, 2, 2))) == [0, 1, 0, 1]


def _create(cfg, compute=0):
    h = C.c_void_p()
    st = _lib.lib().mis_lm_create(json.dumps(cfg).encode(), compute, 0, C.byref(h))
    if st == 0:
        _lib.lib().mis_tts_destroy(h)
    return st, _lib.last_error()


def test_configuration_errors_are_found_before_the_device():
    ok = config([parallel(), lightning()], loop=(0, 1, 2))
    for key in ("width", "vocab", "layers", "norm"):
        st, msg = _create({k: v for k, v in ok.items() if k != key})
        assert st == 3 and key in msg

    def broken(change):
        c = json.loads(json.dumps(ok))
        change(c)
        st, msg = _create(c)
        assert st == 3, msg
        return msg
    for key in ("heads", "kv_heads", "dim", "vdim", "scale"):
        assert key in broken(lambda c: c["layers"][0]["mixer"]["left"].pop(key))
    for key in ("width", "blocks", "conv"):
        assert key in broken(lambda c: c["layers"][0]["mixer"]["right"].pop(key))
    for key in ("left", "right", "left_scale", "right_scale"):
        assert key in broken(lambda c: c["layers"][0]["mixer"].pop(key))
    for key in ("heads", "dim", "vdim", "decay"):
        assert key in broken(lambda c: c["layers"][1]["mixer"].pop(key))
    broken(lambda c: c["layers"][0].update(type="latent_attention"))
    broken(lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=4))
    broken(lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=22))
    broken(lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=7))
    broken(lambda c: c["layers"][0]["mixer"]["right"].update(blocks=4))
    broken(lambda c: c["layers"][1]["mixer"].update(decay=[0.5]))
    broken(lambda c: c["layers"][1]["mixer"].update(decay=[0.5, 0.5, 1.5]))
    broken(lambda c: c["layers"][1]["mlp"].update(kind="mixture"))
    broken(lambda c: c["loop"].update(stop=3))
    broken(lambda c: c["loop"].update(times=0))
    if _lib.lib().mis_device_count() == 0:
        for c in (ok, odd()):
            assert _create(c)[0] == 7                                           # device: no CPU fallback


def test_registry_and_configuration():
    assert registry.model_class({"architecture": "Vamunex"}) is mas.BlockLanguageModel and mas.BlockLanguageModel in registry.FLOAT32
    c = mas.BlockModelConfiguration.from_dict(config([lightning()], loop=(0, 1, 4)))
    assert c.loop == dict(start=0, stop=1, times=4) and c.to_dict()["loop"] == c.loop
    assert mas.BlockModelConfiguration.from_dict(config([parallel(left(), right())])).loop is None
