"""Vamunex - plain numpy restatement (float64, one function per mechanism, no cache, no batching, one token after the other in the recurrences): the
test oracle of the language model that mixes windowed attention, a gated linear recurrence and lightning attention.  Shares no code with the engine.

Notation: T tokens of one sequence, d width.  Weights are dictionaries name -> array in the checkpoint's own [out, in] orientation.

    norm(x; w)     x / sqrt(mean x^2 + eps) * (1 + w)
    x_0            E[token]
    layer          x <- x + norm(mix(norm(x; n1)); n1b);   x <- x + norm(ff(norm(x; n2)); n2b)
    lightning      S_t = c S_{t-1} + k_t v_t^T,  o_t = S_t^T q_t   per head, q, k, v through silu;  W_o (rms(o) * g * sigmoid(W_g h))
    parallel       a * attention(h) + b * recurrence(h)
      attention    grouped heads, normed and rotated q, k; position i sees j <= i with i - j < size or j < keep_first; the softmax's denominator
                   has one more term exp(sink)
      recurrence   u = conv(W_x h), r, g = sigmoid of block-diagonal products of u, a = exp(-8 r softplus(lam)),
                   S_t = a S_{t-1} + sqrt(1 - a^2) g u;  W_o (S * gelu(W_y h))
    ff             W_down (silu(W_gate h) * W_up h)
    logits         head norm(x; n_final)

A range of layers may run several times in a row with the same weights; every pass starts from its own empty cache or state.
"""
from __future__ import annotations

import math

import numpy as np


def f64(a):
    return np.asarray(a, np.float64)


def rms(x, eps):
    x = f64(x)
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def offset_norm(x, w, eps):
    return rms(x, eps) * (1.0 + f64(w))


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-f64(z)))


def silu(z):
    return f64(z) * sigmoid(z)


def gelu_tanh(z):
    z = f64(z)
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def linear(h, w, b=None):
    y = f64(h) @ f64(w).T
    return y if b is None else y + f64(b)


# ---- feed-forward
def gated_feed_forward(h, gate, up, down):
    return linear(silu(linear(h, gate)) * linear(h, up), down)


# ---- lightning attention
def decayed_outer_state(q, k, v, decay):
    """q, k [T, D], v [T, E] of one head -> [T, E]"""
    S = np.zeros((k.shape[1], v.shape[1]))
    out = np.zeros((q.shape[0], v.shape[1]))
    for t in range(q.shape[0]):
        S = decay * S + np.outer(k[t], v[t])
        out[t] = S.T @ q[t]
    return out


def lightning(h, mx, w, eps):
    T, H, D, E = h.shape[0], mx["heads"], mx["dim"], mx["vdim"]
    q, k = silu(linear(h, w["q"])).reshape(T, H, D), silu(linear(h, w["k"])).reshape(T, H, D)
    v = silu(linear(h, w["v"])).reshape(T, H, E)
    o = np.concatenate([decayed_outer_state(q[:, a], k[:, a], v[:, a], mx["decay"][a]) for a in range(H)], axis=1)
    return linear(rms(o, eps) * f64(w["norm"]) * sigmoid(linear(h, w["g"])), w["o"])


# ---- windowed attention with kept first tokens and a sink
def rotate_half(x, positions, dims, base):
    """x [T, ..., D]: pair i = elements (i, i + dims / 2) turned by position * base^(-2 i / dims); elements from dims on pass."""
    x = f64(x)
    y = x.copy()
    n = dims // 2
    for i in range(n):
        a = f64(positions) * base ** (-2.0 * i / dims)
        shape = (len(a),) + (1,) * (x.ndim - 2)
        c, s = np.cos(a).reshape(shape), np.sin(a).reshape(shape)
        u, v = x[..., i], x[..., i + n]
        y[..., i], y[..., i + n] = u * c - v * s, v * c + u * s
    return y


def kept_window_mask(T, size=None, keep_first=0):
    """[T, T] of bool: which keys j a query i sees."""
    m = np.zeros((T, T), bool)
    for i in range(T):
        for j in range(i + 1):
            m[i, j] = size is None or i - j < size or j < keep_first
    return m


def sink_softmax(scores, mask, sink):
    """Weights of the visible keys; the sink takes its share and gives nothing."""
    out = np.zeros_like(scores)
    for i in range(scores.shape[0]):
        z = scores[i, mask[i]]
        top = max(z.max(), sink)
        e = np.exp(z - top)
        out[i, mask[i]] = e / (e.sum() + math.exp(sink - top))
    return out


def attention(h, mx, w, eps):
    T, H, G, D, E = h.shape[0], mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    pos = np.arange(T)
    q = rms(linear(h, w["q"], w["q.b"]).reshape(T, H, D), eps) * f64(w["q.norm"])
    k = rms(linear(h, w["k"], w["k.b"]).reshape(T, G, D), eps) * f64(w["k.norm"])
    v = linear(h, w["v"], w["v.b"]).reshape(T, G, E)
    rot = mx["rot"]
    q, k = rotate_half(q, pos, rot["dims"], rot["base"]), rotate_half(k, pos, rot["dims"], rot["base"])
    mk = mx.get("mask") or {}
    mask = kept_window_mask(T, mk.get("size"), mk.get("keep_first", 0))
    out = np.zeros((T, H, E))
    for a in range(H):
        g = a // (H // G)
        p = sink_softmax((q[:, a] @ k[:, g].T) * mx["scale"], mask, float(w["sink"][a]))
        out[:, a] = p @ v[:, g]
    return linear(out.reshape(T, H * E), w["o"], w["o.b"])


# ---- gated linear recurrence behind a short convolution
def causal_conv(x, taps, bias):
    """x [T, C], taps [C, n] (the last column weighs the current token), zeros before the start."""
    x, taps = f64(x), f64(taps)
    n = taps.shape[1]
    y = np.tile(f64(bias), (x.shape[0], 1))
    for t in range(x.shape[0]):
        for i in range(n):
            if t - i >= 0:
                y[t] += taps[:, n - 1 - i] * x[t - i]
    return y


def block_diagonal(u, w, b):
    """u [T, B * n], w [B, n, n] (out, in), b [B, n]"""
    n = w.shape[1]
    return np.concatenate([linear(u[:, i * n:(i + 1) * n], w[i], b[i]) for i in range(w.shape[0])], axis=1)


def gated_recurrence(u, r, g, lam):
    log_a = -8.0 * f64(r) * np.log1p(np.exp(f64(lam)))
    a = np.exp(log_a)
    S, out = np.zeros(u.shape[1]), np.zeros(u.shape)
    for t in range(u.shape[0]):
        S = a[t] * S + np.sqrt(1.0 - a[t] ** 2) * g[t] * u[t]
        out[t] = S
    return out


def recurrent(h, mx, w):
    y = gelu_tanh(linear(h, w["y"], w["y.b"]))
    u = causal_conv(linear(h, w["x"], w["x.b"]), w["conv"], w["conv.b"])
    r, g = sigmoid(block_diagonal(u, w["ra"], w["ra.b"])), sigmoid(block_diagonal(u, w["ri"], w["ri.b"]))
    return linear(gated_recurrence(u, r, g, w["lam"]) * y, w["o"])


def side(w, name):
    return {k[len(name) + 1:]: v for k, v in w.items() if k.startswith(name + ".")}


def parallel(h, mx, w, eps):
    return mx["left_scale"] * attention(h, mx["left"], side(w, "left"), eps) + mx["right_scale"] * recurrent(h, mx["right"], side(w, "right"))


# ---- the model
def layer_order(cfg):
    n = len(cfg["layers"])
    lp = cfg.get("loop")
    if not lp:
        return list(range(n))
    return list(range(lp["start"])) + list(range(lp["start"], lp["stop"])) * lp["times"] + list(range(lp["stop"], n))


def forward(cfg, W, tokens, return_layers=False):
    """cfg: config.json as a dictionary, W: name -> array, tokens: the ids of one sequence.  -> logits [T, vocab] (and the residual stream behind
    every layer run)."""
    eps = cfg["norm"]["eps"]
    x = f64(W["embed"])[np.asarray(tokens)]
    runs = []
    for i in layer_order(cfg):
        L, w = cfg["layers"][i], side(W, f"l{i}")
        mix = side(w, "mix")
        h = offset_norm(x, w["norm1"], eps)
        y = lightning(h, L["mixer"], mix, eps) if L["type"] == "lightning" else parallel(h, L["mixer"], mix, eps)
        x = x + offset_norm(y, w["norm1b"], eps)
        if L.get("mlp") is not None:
            y = gated_feed_forward(offset_norm(x, w["norm2"], eps), w["mlp.gate"], w["mlp.up"], w["mlp.down"])
            x = x + offset_norm(y, w["norm2b"], eps)
        runs.append(x)
    out = linear(offset_norm(x, W["final.norm"], eps), W["head"])
    return (out, runs) if return_layers else out


# ---- random models for the tests -----------------------------------------------------------------------------------------------------
def to_bf16(a):
    """Round to the nearest bfloat16 (ties to even), as float32."""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    u = (u + 0x7FFF + ((u >> 16) & 1)) & np.uint32(0xFFFF0000)
    return u.view(np.float32)


def random_weights(cfg, seed=0, branch=0.4):
    """bfloat16-representable float32 arrays for every tensor `cfg` implies.  `branch`: size of what a sublayer adds to the stream."""
    g = np.random.default_rng(seed)
    d, V = cfg["width"], cfg["vocab"]

    def mat(n, k, a=1.0):
        return to_bf16(g.standard_normal((n, k)) * (a / math.sqrt(k)))

    def vec(n, around=0.0, spread=0.2):
        return to_bf16(around + spread * g.standard_normal(n))
    W = {"embed": to_bf16(g.standard_normal((V, d))), "final.norm": vec(d), "head": mat(V, d, 4.0)}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        W[p + "norm1"], W[p + "norm1b"] = vec(d), vec(d, branch - 1.0, 0.1)
        if L.get("mlp") is not None:
            ff = L["mlp"]["ff"]
            W[p + "norm2"], W[p + "norm2b"] = vec(d), vec(d, branch - 1.0, 0.1)
            W[p + "mlp.gate"], W[p + "mlp.up"], W[p + "mlp.down"] = mat(ff, d), mat(ff, d), mat(d, ff)
        p += "mix."
        if L["type"] == "lightning":
            HD, HE = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            W[p + "q"], W[p + "k"], W[p + "v"], W[p + "g"] = mat(HD, d), mat(HD, d), mat(HE, d), mat(HE, d)
            W[p + "norm"], W[p + "o"] = vec(HE, 1.0), mat(d, HE)
            continue
        a, p0 = m["left"], p + "left."
        H, G, D, E = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
        for n, rows in (("q", H * D), ("k", G * D), ("v", G * E)):
            W[p0 + n], W[p0 + n + ".b"] = mat(rows, d), vec(rows)
        W[p0 + "q.norm"], W[p0 + "k.norm"] = vec(D, 1.4), vec(D, 1.0)
        W[p0 + "sink"] = vec(H, 0.5, 1.0)
        W[p0 + "o"], W[p0 + "o.b"] = mat(d, H * E), vec(d)
        r, p1 = m["right"], p + "right."
        w, B, n = r["width"], r["blocks"], r["width"] // r["blocks"]
        for nm in ("y", "x"):
            W[p1 + nm], W[p1 + nm + ".b"] = mat(w, d), vec(w)
        W[p1 + "conv"], W[p1 + "conv.b"] = vec((w, r["conv"]), 0.0, 0.6), vec(w)
        for nm in ("ra", "ri"):
            W[p1 + nm] = to_bf16(g.standard_normal((B, n, n)) / math.sqrt(n))
            W[p1 + nm + ".b"] = vec((B, n))
        W[p1 + "lam"] = vec(w, -3.5, 1.5)                                       # from a memory of a few tokens to one of hundreds
        W[p1 + "o"] = mat(d, w, 1.5)
    return W
