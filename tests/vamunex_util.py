"""Small Vamunex configurations and helpers shared by the tests."""
import math

import numpy as np

from oracle import vamunex as orc
from rugunex_util import rel_rms, row_rel_rms  # noqa: F401


def lightning(heads=3, dim=18, vdim=30, decay=None, mlp=136):
    decay = decay or [1.0 - 0.6 ** (a + 1) for a in range(heads)]
    return dict(type="lightning", mixer=dict(heads=heads, dim=dim, vdim=vdim, decay=list(decay)), mlp=mlp and dict(kind="dense", ff=mlp))


def left(heads=6, kv_heads=2, dim=20, vdim=28, window=17, keep=3, rot=12, base=700.0, scale=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale if scale is not None else 1.3 / math.sqrt(dim), rot=dict(base=base, dims=rot))
    if window is not None:
        m["mask"] = dict(size=window, keep_first=keep)
    return m


def right(width=105, blocks=5, conv=3):
    return dict(width=width, blocks=blocks, conv=conv)


def parallel(lf=None, rt=None, left_scale=0.8, right_scale=1.3, mlp=136):
    return dict(type="parallel", mixer=dict(left=lf or left(), right=rt or right(), left_scale=left_scale, right_scale=right_scale),
                mlp=mlp and dict(kind="dense", ff=mlp))


def config(layers, width=184, vocab=301, eps=3e-6, loop=None):
    c = dict(architecture="Vamunex", width=width, vocab=vocab, layers=layers, norm=dict(eps=eps))
    if loop:
        c["loop"] = dict(start=loop[0], stop=loop[1], times=loop[2])
    return c


def odd():
    """Sizes that are multiples of nothing, layers without feed-forward, layers that run three times."""
    return config([parallel(), lightning(), parallel(left(heads=4, kv_heads=4, dim=34, vdim=10, rot=2, window=29, keep=0), right(33, 3, 5), mlp=None),
                   lightning(heads=2, dim=70, vdim=65, mlp=None)], loop=(1, 3, 3))


def wide():
    """The heads of a large model in a narrow one."""
    return config([lightning(heads=4, dim=128, vdim=128, mlp=520), parallel(left(heads=16, kv_heads=2, dim=128, vdim=128, window=150, keep=5, rot=128, base=1e5),
                                                                             right(512, 2, 4), mlp=520)], width=320, vocab=1000, loop=(0, 1, 2))


def groups():
    """More query heads per key head than a matrix tile holds, values wider than keys, one block in the recurrence, no convolution to speak of."""
    return config([parallel(left(heads=40, kv_heads=2, dim=64, vdim=96, window=90, keep=1, rot=64), right(96, 1, 1), mlp=70),
                   lightning(heads=5, dim=96, vdim=160, mlp=300)], width=136, vocab=120)


def full():
    """Every key visible, as many key heads as query heads, one channel per block, a long convolution, decays of 0 and 1."""
    return config([parallel(left(heads=3, kv_heads=3, dim=160, vdim=200, window=None, rot=40), right(48, 48, 6)),
                   lightning(heads=3, dim=33, vdim=64, decay=[0.0, 1.0, 0.97]),
                   parallel(left(heads=2, kv_heads=1, dim=8, vdim=16, window=64, keep=64, rot=0), right(640, 2, 2))], width=100, vocab=90, loop=(0, 2, 1))


def huge():
    """Past what the matrix-core kernels take: the general kernels."""
    return config([parallel(left(heads=2, kv_heads=1, dim=300, vdim=290, window=33, keep=2, rot=30), right(600, 1, 4), mlp=90),
                   lightning(heads=2, dim=290, vdim=70, mlp=90)], width=150, vocab=100)


def without(W, which):
    """The weights with one sublayer switched off everywhere: 'norm1b' the mixers, 'norm2b' the feed-forwards."""
    return {k: (np.full_like(v, -1.0) if k.endswith("." + which) else v) for k, v in W.items()}


def one_side(cfg, which):
    """Only one side of every parallel mixer."""
    out = dict(cfg, layers=[])
    for L in cfg["layers"]:
        if L["type"] == "parallel":
            L = dict(L, mixer=dict(L["mixer"], **{("right_scale" if which == "left" else "left_scale"): 0.0}))
        out["layers"].append(L)
    return out


def standout(cfg, W, key_token, query_token, gain=30.0):
    """Layer 0 reads the tokens themselves, so both vectors are known: query_token's query is made to point along key_token's key in the dimensions
    that do not turn with the position, in every head; no other query does."""
    eps, mx = cfg["norm"]["eps"], cfg["layers"][0]["mixer"]["left"]
    H, G, D, rot = mx["heads"], mx["kv_heads"], mx["dim"], mx["rot"]["dims"]
    W = dict(W)
    p = "l0.mix.left."
    for n in ("q", "k"):
        W[p + n + ".b"] = np.zeros_like(W[p + n + ".b"])
        W[p + n + ".norm"] = np.ones_like(W[p + n + ".norm"])
    h = orc.offset_norm(W["embed"][[key_token, query_token]], W["l0.norm1"], eps)
    k = (h[0] @ W[p + "k"].T.astype(np.float64)).reshape(G, D)
    k[:, :rot] = 0.0
    q = W[p + "q"].astype(np.float64).reshape(H, D, -1).copy()
    for a in range(H):
        q[a] += gain * np.outer(k[a // (H // G)], h[1]) / (h[1] @ h[1])
    W[p + "q"] = orc.to_bf16(q.reshape(H * D, -1))
    W["l0.mix.left.sink"] = orc.to_bf16(np.zeros(H))
    return W
