"""Small Rugunex configurations and helpers shared by the tests."""
import math

import numpy as np

from oracle import rugunex as orc

YARN = dict(factor=5.0, original=96, fast=24.0, slow=1.5)


def mixer(heads=5, dim=24, rot_dim=10, vdim=20, kv_rank=72, window=17, scale=None, base=3000.0, scaling=YARN):
    m = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, scale=scale if scale is not None else 0.9 / math.sqrt(dim + rot_dim),
             rot=dict(base=base, dims=rot_dim))
    if window is not None:
        m["mask"] = dict(size=window)
    if scaling is not None:
        m["rot"]["scaling"] = dict(scaling)
    return m


def config(width=200, vocab=333, layers=None, ff=136, eps=2e-6, logit_scale=0.7, logit_softcap=25.0):
    layers = layers or [dict(mixer=mixer())]
    out = []
    for e in layers:
        e = dict(e)
        e.setdefault("mlp", dict(kind="dense", ff=ff))
        out.append(dict(type="latent_attention", **e))
    return dict(architecture="Rugunex", width=width, vocab=vocab, layers=out, norm=dict(eps=eps), logit_scale=logit_scale, logit_softcap=logit_softcap)


def odd():
    """Sizes that are multiples of nothing; a layer without feed-forward, a shared layer, windows that differ."""
    return config(layers=[dict(mixer=mixer()), dict(mixer=mixer(heads=3, dim=40, vdim=33, kv_rank=50, rot_dim=6, window=29, base=50.0), mlp=None),
                          dict(mixer=mixer(), weights_of=0), dict(mixer=mixer(window=1, scaling=None), mlp=dict(kind="dense", ff=70))])


def wide():
    """The sizes of a large model's attention in a narrow model: two tiles of heads, 512 + 64 cached values."""
    return config(width=320, vocab=1000, ff=520, layers=[dict(mixer=mixer(heads=20, dim=128, rot_dim=64, vdim=128, kv_rank=512, window=150, base=1e5,
                                                                          scaling=dict(factor=8.0, original=128, fast=32.0, slow=1.0)))] * 2)


def middle():
    """256 latent values, values wider than keys, every key visible."""
    return config(width=264, vocab=257, ff=300, layers=[dict(mixer=mixer(heads=17, dim=96, rot_dim=32, vdim=200, kv_rank=256, window=None, scaling=None)),
                                                        dict(mixer=mixer(heads=2, dim=160, rot_dim=62, vdim=64, kv_rank=200, window=70))])


def many():
    """More heads than one attention block takes; more value tiles than waves, a latent that is no multiple of 512."""
    return config(width=136, vocab=120, ff=100, layers=[dict(mixer=mixer(heads=37, dim=8, rot_dim=4, vdim=12, kv_rank=40, window=90)),
                                                        dict(mixer=mixer(heads=12, dim=64, rot_dim=32, vdim=136, kv_rank=448, window=130))])


def huge():
    """Past what the matrix-core attention kernels take: the general kernels."""
    return config(width=150, vocab=100, ff=90, layers=[dict(mixer=mixer(heads=3, dim=250, rot_dim=20, vdim=30, kv_rank=70, window=40)),
                                                       dict(mixer=mixer(heads=2, dim=30, rot_dim=8, vdim=300, kv_rank=600, window=33))])


def no_branch(W, which):
    """The weights with one branch switched off everywhere ('ls1' the mixers, 'ls2' the feed-forwards)."""
    return {k: (np.zeros_like(v) if k.endswith("." + which) else v) for k, v in W.items()}


def standout(cfg, W, layer, key_token, query_token, gain):
    """Adds to W_q of layer 0 what makes query_token's unrotated query point along key_token's unrotated key in every head: its score with that key
    stands out by about `gain` (layer 0 reads the tokens themselves, so both vectors are known)."""
    assert layer == 0
    eps, mx = cfg["norm"]["eps"], cfg["layers"][0]["mixer"]
    w = orc.layer_weights(W, 0)
    h = orc.rms_norm(orc.rms_norm(W["embed"][[key_token, query_token]].astype(np.float64), W["embed.norm"], eps), w["norm1"], eps)
    H, n, r = mx["heads"], mx["dim"], mx["rot_dim"]
    c, _ = orc.latent(h, w["mix.dkv"], w["mix.dkv.norm"], mx["kv_rank"], eps)
    k = (c[0] @ w["mix.uk"].T.astype(np.float64)).reshape(H, n)
    q = W["l0.mix.q"].astype(np.float64).reshape(H, n + r, -1).copy()
    for a in range(H):
        q[a, :n] += gain / (mx["scale"] * (k[a] @ k[a])) * np.outer(k[a], h[1]) / (h[1] @ h[1])
    W = dict(W)
    W["l0.mix.q"] = orc.to_bf16(q.reshape(H * (n + r), -1))
    return W


def rel_rms(got, ref):
    got, ref = np.asarray(got, np.float64), np.asarray(ref, np.float64)
    return float(np.sqrt(np.mean((got - ref) ** 2)) / np.sqrt(np.mean((ref - ref.mean(-1, keepdims=True)) ** 2)))


def row_rel_rms(got, ref):
    """The largest over the rows."""
    ref = np.asarray(ref, np.float64)
    scale = np.sqrt(np.mean((ref - ref.mean(-1, keepdims=True)) ** 2))
    return float(np.sqrt(np.mean((np.asarray(got, np.float64) - ref) ** 2, axis=-1)).max() / scale)
