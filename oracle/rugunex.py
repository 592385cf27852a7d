"""Rugunex - plain numpy restatement (float64, one function per mechanism, no cache, no batching): the test oracle of the parallel-block
latent-attention language model.  Shares no code with the engine.

Notation: T tokens of one sequence, d width, H heads; per head n unrotated and r rotated query / key dimensions, v value dimensions;
R latent size.  Weights are dictionaries name -> array in the checkpoint's own [out, in] orientation.

    x_0      = rms(E[token]) * g_embed
    layer    h = rms(x) * g1;   x <- x + s1 * mix(h) + s2 * ff(h)            (one norm, both branches read it)
    mix(h)   q = W_q h (per head: n plain, r rotary);  [c_raw | k_r] = W_dkv h;  c = rms(c_raw) * g_c
             score(i, j) = (q_i . (W_uk c_j) + rot(q_i) . rot(k_r_j)) * scale     for 0 <= i - j < window
             out_i = W_o concat_h( sum_j softmax_j * W_uv c_j )
    ff(h)    W_down relu(W_up h)^2
    logits   cap * tanh( (head (rms(x) * g_final)) * logit_scale / cap )
"""
from __future__ import annotations

import math

import numpy as np


def rms_norm(x, w, eps):
    x = np.asarray(x, np.float64)
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * np.asarray(w, np.float64)


def relu_squared(z):
    z = np.maximum(np.asarray(z, np.float64), 0.0)
    return z * z


def feed_forward(h, up, down):
    return relu_squared(h @ np.asarray(up, np.float64).T) @ np.asarray(down, np.float64).T


def rotary_frequencies(dims, base, scaling=None):
    """Angle per position of each rotated pair.  `scaling` (YaRN): pairs that turn more than `fast` times over the original context keep
    their frequency, pairs that turn less than `slow` times get it divided by `factor`, the ones between are blended linearly."""
    f = np.asarray([base ** (-2.0 * i / dims) for i in range(dims // 2)], np.float64)
    if scaling is None:
        return f
    fac, orig = float(scaling["factor"]), float(scaling["original"])

    def turns_to_dim(turns):
        return dims * math.log(orig / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(turns_to_dim(scaling["fast"])), 0)
    hi = min(math.ceil(turns_to_dim(scaling["slow"])), dims - 1)
    ramp = np.asarray([min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(dims // 2)])
    return f / fac * ramp + f * (1.0 - ramp)


def rotary_magnitude(scaling=None):
    return 1.0 if scaling is None else 0.1 * math.log(float(scaling["factor"])) + 1.0


def rotate_interleaved(x, positions, freqs, magnitude=1.0):
    """x [T, ..., D]: pair i = elements (2i, 2i + 1) turned by positions * freqs[i]; elements past the pairs pass through."""
    x = np.asarray(x, np.float64)
    y = x.copy()
    ang = np.asarray(positions, np.float64)[:, None] * freqs[None, :]
    shape = (ang.shape[0],) + (1,) * (x.ndim - 2) + (ang.shape[1],)
    c, s = (np.cos(ang) * magnitude).reshape(shape), (np.sin(ang) * magnitude).reshape(shape)
    n = 2 * len(freqs)
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    y[..., 0:n:2] = u * c - v * s
    y[..., 1:n:2] = v * c + u * s
    return y


def window_mask(T, size):
    """[T, T] of bool: query i sees keys i - size + 1 .. i (size None: every key up to i)."""
    m = np.zeros((T, T), bool)
    for i in range(T):
        m[i, max(0, i - size + 1 if size else 0): i + 1] = True
    return m


def masked_softmax(scores, mask):
    out = np.zeros_like(scores)
    for i in range(scores.shape[0]):
        z = scores[i, mask[i]]
        e = np.exp(z - z.max())
        out[i, mask[i]] = e / e.sum()
    return out


def latent(h, w_dkv, norm_w, rank, eps):
    """-> (c [T, rank] normed latent, k_r [T, rot_dim] shared key part before the rotation)"""
    y = h @ np.asarray(w_dkv, np.float64).T
    return rms_norm(y[:, :rank], norm_w, eps), y[:, rank:]


def latent_attention(h, mx, w, eps, positions=None):
    """h [T, d] -> [T, d].  mx: the layer's mixer entry of config.json; w: {'q', 'dkv', 'dkv.norm', 'uk', 'uv', 'o'}."""
    T = h.shape[0]
    H, n, r, v, R = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
    pos = np.arange(T) if positions is None else positions
    q = (h @ np.asarray(w["q"], np.float64).T).reshape(T, H, n + r)
    c, k_r = latent(h, w["dkv"], w["dkv.norm"], R, eps)
    rot = mx["rot"]
    freqs, mag = rotary_frequencies(rot["dims"], rot["base"], rot.get("scaling")), rotary_magnitude(rot.get("scaling"))
    q_r = rotate_interleaved(q[:, :, n:], pos, freqs, mag)
    k_r = rotate_interleaved(k_r, pos, freqs, mag)
    k = (c @ np.asarray(w["uk"], np.float64).T).reshape(T, H, n)
    val = (c @ np.asarray(w["uv"], np.float64).T).reshape(T, H, v)
    mask = window_mask(T, (mx.get("mask") or {}).get("size"))
    out = np.zeros((T, H, v))
    for a in range(H):
        s = (q[:, a, :n] @ k[:, a].T + q_r[:, a] @ k_r.T) * mx["scale"]
        out[:, a] = masked_softmax(s, mask) @ val[:, a]
    return out.reshape(T, H * v) @ np.asarray(w["o"], np.float64).T


def output_logits(x, final_norm, head, eps, logit_scale, softcap):
    z = rms_norm(x, final_norm, eps) @ np.asarray(head, np.float64).T * logit_scale
    return softcap * np.tanh(z / softcap)


def layer_weights(W, i):
    p = f"l{i}."
    return {k[len(p):]: v for k, v in W.items() if k.startswith(p)}


def forward(cfg, W, tokens, return_layers=False):
    """cfg: config.json as a dictionary, W: name -> array, tokens: the ids of one sequence.  -> logits [T, vocab] (and the residual
    stream after every layer)."""
    eps = cfg["norm"]["eps"]
    x = rms_norm(np.asarray(W["embed"], np.float64)[np.asarray(tokens)], W["embed.norm"], eps)
    layers = []
    for i, L in enumerate(cfg["layers"]):
        w = layer_weights(W, L.get("weights_of", i) if L.get("weights_of") is not None else i)
        h = rms_norm(x, w["norm1"], eps)
        y = np.asarray(w["ls1"], np.float64) * latent_attention(h, L["mixer"], {k[4:]: a for k, a in w.items() if k.startswith("mix.")}, eps)
        if L.get("mlp") is not None:
            y = y + np.asarray(w["ls2"], np.float64) * feed_forward(h, w["mlp.up"], w["mlp.down"])
        x = x + y
        layers.append(x)
    out = output_logits(x, W["final.norm"], W["head"], eps, cfg["logit_scale"], cfg["logit_softcap"])
    return (out, layers) if return_layers else out


# ---- random models for the tests -----------------------------------------------------------------------------------------------------
def to_bf16(a):
    """Round to the nearest bfloat16 (ties to even), as float32."""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    u = (u + 0x7FFF + ((u >> 16) & 1)) & np.uint32(0xFFFF0000)
    return u.view(np.float32)


def random_weights(cfg, seed=0, branch=0.6):
    """bfloat16-representable float32 arrays for every tensor `cfg` implies.  `branch`: size of the two branches' layer scales."""
    g = np.random.default_rng(seed)
    d, V = cfg["width"], cfg["vocab"]

    def mat(n, k, a=1.0):
        return to_bf16(g.standard_normal((n, k)) * (a / math.sqrt(k)))

    def vec(n, around=1.0, spread=0.2):
        return to_bf16(around + spread * g.standard_normal(n))
    W = {"embed": to_bf16(g.standard_normal((V, d))), "embed.norm": vec(d), "final.norm": vec(d), "head": mat(V, d, 6.0)}
    for i, L in enumerate(cfg["layers"]):
        if L.get("weights_of") is not None:
            continue
        m, p = L["mixer"], f"l{i}."
        H, R, r = m["heads"], m["kv_rank"], m["rot_dim"]
        W[p + "norm1"] = vec(d)
        W[p + "mix.q"] = mat(H * (m["dim"] + r), d, 1.6)
        W[p + "mix.dkv"] = mat(R + r, d, 1.6)
        W[p + "mix.dkv.norm"] = vec(R)
        W[p + "mix.uk"] = mat(H * m["dim"], R)
        W[p + "mix.uv"] = mat(H * m["vdim"], R)
        W[p + "mix.o"] = mat(d, H * m["vdim"])
        W[p + "ls1"] = vec(d, branch)
        if L.get("mlp") is not None:
            W[p + "mlp.up"] = mat(L["mlp"]["ff"], d)
            W[p + "mlp.down"] = mat(d, L["mlp"]["ff"])
            W[p + "ls2"] = vec(d, branch)
    return W
