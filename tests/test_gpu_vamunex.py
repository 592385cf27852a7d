"""Vamunex on the device against oracle/vamunex.py: each mechanism alone (the other sublayers' outer norms are zero, or one side's scale is; compared
in the residual stream behind every layer run), prompts against token-by-token decoding, portions, batches, rows used again, edges of windows and kept
tokens with scores that stand out, memory of the recurrences, and generation through the engine's own loop - in bfloat16 and in the 32-bit mode."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import mlx_audio_swift_amd as mas
from oracle import vamunex as orc
from vamunex_util import config, full, groups, huge, left, lightning, odd, one_side, parallel, right, row_rel_rms, standout, wide, without
from gpu_util import observe

pytestmark = pytest.mark.gpu
# relative rms error of the worst row (mean taken off the reference)
TOL = {"float32": 6e-6, "bfloat16": 2.2e-2}
SHAPES = {"odd": odd, "wide": wide, "groups": groups, "full": full, "huge": huge}
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
both = pytest.mark.parametrize("compute", ["float32", "bfloat16"])


def tokens(n, vocab, seed=0):
    return np.random.default_rng(seed).integers(0, vocab, n).astype(np.int32)


def build(cfg, compute, seed=11):
    W = orc.random_weights(cfg, seed)
    return W, mas.BlockLanguageModel.from_weights(cfg, W, compute=compute)


def run_all(m, toks, cut=None, row=0):
    """Logits of every position, the tokens fed in portions of the sizes in `cut` (the last one repeats)."""
    cut = cut or [len(toks)]
    out, at, k = [], 0, 0
    while at < len(toks):
        n = min(cut[min(k, len(cut) - 1)], len(toks) - at)
        out.append(m.extend([(row, toks[at:at + n])], [list(range(n))]))
        at += n; k += 1
    return np.concatenate(out)


def check(got, ref, compute, kind="logits", factor=1.0):
    assert np.isfinite(got).all()
    assert observe(f"vamunex_{kind}_{compute}", row_rel_rms(got, ref), TOL[compute] * factor)


# ---------------------------------------------------------------- mechanisms alone
@both
@pytest.mark.parametrize("alone", ["stream", "mlp", "left", "right", "mixers"])
@pytest.mark.parametrize("shape", list(SHAPES))
def test_mechanism_alone(shape, alone, compute):
    cfg = SHAPES[shape]()
    W = orc.random_weights(cfg, 2)
    if alone in ("stream", "mlp"):
        W = without(W, "norm1b")
    if alone != "mlp":
        W = without(W, "norm2b")
    if alone in ("left", "right"):
        cfg = one_side(cfg, alone)
    m = mas.BlockLanguageModel.from_weights(cfg, W, compute=compute)
    t = tokens(150, cfg["vocab"], 3)
    m.reset(1, 160)
    got, res = m.extend([(0, t)], [list(range(150))], return_residual=True)
    ref, layers = orc.forward(cfg, W, t, return_layers=True)
    assert len(res) == len(layers) == len(orc.layer_order(cfg))
    if alone == "stream":
        assert np.abs(res[-1] - layers[-1]).max() < 1e-5 * np.abs(layers[-1]).max()          # a float32 stream in both modes
    for a, b in zip(res, layers):
        check(a, b, compute, alone)
    check(got, ref, compute)


@both
def test_sink_takes_its_share(compute):
    """Sinks far above and far below every score."""
    cfg = config([parallel(left(heads=4, kv_heads=2, dim=32, vdim=32, window=24, keep=2, rot=32), mlp=None)], width=128, vocab=64)
    cfg = one_side(cfg, "left")
    W = orc.random_weights(cfg, 4)
    W["l0.mix.left.o.b"] = np.zeros_like(W["l0.mix.left.o.b"])
    W["l0.mix.left.v.b"] = np.full_like(W["l0.mix.left.v.b"], 1.0)
    t = tokens(90, 64, 5)
    base = None
    for sink in ([-40.0] * 4, [6.0, -3.0, 2.0, 9.0]):
        W["l0.mix.left.sink"] = orc.to_bf16(np.asarray(sink))
        ref = orc.forward(cfg, W, t)
        if base is not None:
            assert np.abs(ref - base).max() > 0.5
        base = ref
        m = mas.BlockLanguageModel.from_weights(cfg, W, compute=compute)
        for cut in ([90], [40, 1]):
            m.reset(1, 96)
            check(run_all(m, t, cut), ref, compute, "sink")


# ---------------------------------------------------------------- whole prompts, portions, decoding
@both
@pytest.mark.parametrize("shape", list(SHAPES))
def test_prompt_portions_and_decoding(shape, compute):
    """One pass, passes of a few rows, portions down to two tokens, and token by token - all against the oracle."""
    cfg = SHAPES[shape]()
    W, m = build(cfg, compute)
    n = 330 if shape == "wide" else 200
    t = tokens(n, cfg["vocab"], 5)
    ref = orc.forward(cfg, W, t)
    for cut, rows in (([n], 4096), ([n], 50), ([n], 64), ([64, 33, 65, 2], 4096), ([63, 129, 3, 1], 4096), ([2], 4096), ([n - 40, 1], 4096), ([1], 4096)):
        m.set_prefill_rows(rows)
        m.reset(1, n)
        got = run_all(m, t, cut)
        assert np.isfinite(got).all()
        assert observe(f"vamunex_cut{cut[0]}_{rows}_{compute}", row_rel_rms(got, ref), TOL[compute]), (cut, rows)


@both
def test_long_decoding(compute):
    """Many windows and memories past the prompt."""
    cfg = config([parallel(left(heads=2, kv_heads=1, dim=16, vdim=16, window=100, keep=7, rot=16), right(64, 4, 4), mlp=64),
                  lightning(heads=2, dim=16, vdim=16, decay=[0.9, 0.999], mlp=64)], width=128, vocab=97)
    W, m = build(cfg, compute)
    t = tokens(700, 97, 6)
    m.reset(1, 700)
    check(run_all(m, t, [5, 1]), orc.forward(cfg, W, t), compute, "long")


@both
@pytest.mark.parametrize("shape", ["odd", "wide", "groups"])
def test_batch_of_unequal_requests(shape, compute):
    """Prompts of different lengths in one batch, decoded together while the short ones end: every row as if it were alone."""
    cfg = SHAPES[shape]()
    W, m = build(cfg, compute)
    lens, extra = [1, 77, 2, 160, 33], [30, 5, 0, 12, 30]
    seqs = [tokens(a + b, cfg["vocab"], 20 + i) for i, (a, b) in enumerate(zip(lens, extra))]
    for rows in (4096, 70):
        m.set_prefill_rows(rows)
        m.reset(len(lens), 200)
        out = [[] for _ in lens]
        got = m.extend([(b, s[:n]) for b, (s, n) in enumerate(zip(seqs, lens))], [list(range(n)) for n in lens])
        at = 0
        for b, n in enumerate(lens):
            out[b].append(got[at:at + n]); at += n
        for k in range(max(extra)):
            live = [b for b in range(len(lens)) if k < extra[b]]
            got = m.extend([(b, seqs[b][lens[b] + k:lens[b] + k + 1]) for b in reversed(live)])      # (any order of rows)
            for i, b in enumerate(reversed(live)):
                out[b].append(got[i:i + 1])
        for b, s in enumerate(seqs):
            check(np.concatenate(out[b]), orc.forward(cfg, W, s), compute, "batch")
    m.reset(1, 200)
    check(np.concatenate(out[3]), run_all(m, seqs[3], [lens[3], 1]), compute, "alone")               # the same request alone


@both
def test_portions_of_several_requests(compute):
    """Requests that go on in portions beside each other, one of them sitting a pass out: states and histories stay with their row."""
    cfg = odd()
    W, m = build(cfg, compute)
    seqs = [tokens(120, cfg["vocab"], 50 + b) for b in range(3)]
    m.reset(3, 128)
    at, out = [0, 0, 0], [[], [], []]
    for take in ((40, 2, 0), (0, 3, 70), (1, 64, 2), (70, 0, 1), (1, 1, 1), (2, 2, 2), (6, 48, 44)):
        live = [b for b in (2, 0, 1) if take[b]]
        got = m.extend([(b, seqs[b][at[b]:at[b] + take[b]]) for b in live], [list(range(take[b])) for b in live])
        i = 0
        for b in live:
            out[b].append(got[i:i + take[b]]); i += take[b]; at[b] += take[b]
    assert at == [120, 120, 120]
    for b in range(3):
        check(np.concatenate(out[b]), orc.forward(cfg, W, seqs[b]), compute, "beside")


@both
def test_rows_used_again(compute):
    """A reset gives the rows back: nothing of an earlier, longer request shows in what comes after it, at the same and at other batch sizes."""
    cfg = odd()
    W, m = build(cfg, compute)
    a, b = tokens(120, cfg["vocab"], 7), tokens(31, cfg["vocab"], 8)
    ref = orc.forward(cfg, W, b)
    m.reset(2, 128)
    m.extend([(0, a), (1, a[::-1])], [[], []])
    for batch, row, cut in ((2, 1, [20, 1]), (2, 0, [1]), (1, 0, [31]), (3, 2, [20, 1]), (2, 1, [2])):
        m.reset(batch, 128)
        check(run_all(m, b, cut, row=row), ref, compute, "again")


@both
def test_more_rows_than_one_tile(compute):
    cfg = config([parallel(left(heads=2, kv_heads=1, dim=16, vdim=8, window=6, keep=1, rot=4), right(40, 2, 3), mlp=64), lightning(heads=2, dim=8, vdim=24, mlp=64)],
                 width=96, vocab=64)
    W, m = build(cfg, compute)
    seqs = [tokens(3 + b % 5 + 4, 64, b) for b in range(64)]
    m.reset(64, 16)
    m.extend([(b, s[:-4]) for b, s in enumerate(seqs)], [[] for _ in seqs])
    outs = [m.extend([(b, s[len(s) - 4 + k:len(s) - 4 + k + 1]) for b, s in enumerate(seqs)]) for k in range(4)]
    for b, s in enumerate(seqs):
        check(np.stack([o[b] for o in outs]), orc.forward(cfg, W, s)[-4:], compute, "rows")


# ---------------------------------------------------------------- edges that show
def edge_model(window, keep, compute):
    cfg = one_side(config([parallel(left(heads=4, kv_heads=2, dim=32, vdim=32, window=window, keep=keep, rot=4, scale=0.7), mlp=None)], width=256, vocab=80), "left")
    W = standout(cfg, orc.random_weights(cfg, 9), key_token=70, query_token=71)
    return cfg, W, mas.BlockLanguageModel.from_weights(cfg, W, compute=compute)


def edge_case(cfg, W, m, base, q, j, seen, compute):
    """One key that stands out at position j for the query at position q."""
    t = base[:q + 1].copy()
    t[q], t[j] = 71, 70
    ref = orc.forward(cfg, W, t)
    plain = t.copy(); plain[j] = base[j]
    moved = np.abs(ref[q] - orc.forward(cfg, W, plain)[q]).max()
    assert moved > 1.0 if seen else moved < 1e-9
    for cut, rows in (([q + 1], 4096), ([q + 1], 37), ([q, 1], 4096), ([max(j, 1), 2], 4096), ([max(q - 3, 1), 1], 4096)):
        m.set_prefill_rows(rows)
        m.reset(1, 256)
        check(run_all(m, t, cut)[q:], ref[q:], compute, "edge", 1.5)


@both
@pytest.mark.parametrize("window", [1, 2, 31, 32, 33, 64, 65, 150])
def test_window_edge(window, compute):
    """The key just inside the window decides the output, just outside it must not - wherever the edge falls in a tile of keys, a portion, a pass,
    and in decoding."""
    cfg, W, m = edge_model(window, 0, compute)
    base = tokens(240, 70, 10)
    for q in (window + 3, 191, 224):
        if window > 1:
            edge_case(cfg, W, m, base, q, q - window + 1, True, compute)
        edge_case(cfg, W, m, base, q, q - window, False, compute)


@both
@pytest.mark.parametrize("keep", [1, 5, 16, 31, 32, 33, 64, 70])
def test_kept_first_tokens(keep, compute):
    """The last kept token is seen from anywhere, the one behind it only through the window; kept tokens and a window that still reaches them."""
    window = 20
    cfg, W, m = edge_model(window, keep, compute)
    base = tokens(240, 70, 11)
    for q in (keep + window + 7, 190):
        edge_case(cfg, W, m, base, q, keep - 1, True, compute)
        edge_case(cfg, W, m, base, q, 0, True, compute)
        edge_case(cfg, W, m, base, q, keep, False, compute)
    edge_case(cfg, W, m, base, keep + window - 1, keep, True, compute)          # kept tokens and window meet
    edge_case(cfg, W, m, base, keep + window, keep, False, compute)             # a gap of one token between them


@both
def test_far_key_among_hundreds(compute):
    """No window: one key far back stands out, in a prompt and in decoding (key shares meet over 400 keys)."""
    cfg, W, m = edge_model(None, 0, compute)
    for key in (0, 1, 31, 32, 255, 398):
        t = tokens(400, 70, 13)
        t[key], t[399] = 70, 71
        ref = orc.forward(cfg, W, t)
        for cut in ([400], [399, 1], [70, 329, 1]):
            m.reset(1, 400)
            check(run_all(m, t, cut)[399:], ref[399:], compute, "far", 1.5)


@both
def test_recurrent_memory_reaches_far(compute):
    """States that hardly fade: the first tokens still show hundreds of tokens later, whatever the portions - the carried state decides the logits."""
    cfg = config([parallel(left(window=8, keep=0), right(64, 2, 4), mlp=None), lightning(heads=2, dim=32, vdim=32, decay=[1.0, 0.9995], mlp=None)], width=96, vocab=64)
    W = orc.random_weights(cfg, 14)
    W["l0.mix.right.lam"] = orc.to_bf16(np.full(64, -9.0))
    t = tokens(500, 64, 15)
    ref = orc.forward(cfg, W, t)
    t2 = t.copy(); t2[:200] = tokens(200, 64, 16)
    assert np.abs(ref[-1] - orc.forward(cfg, W, t2)[-1]).max() > 0.5
    m = mas.BlockLanguageModel.from_weights(cfg, W, compute=compute)
    for cut, rows in (([500], 4096), ([500], 33), ([64, 65, 1], 4096), ([440, 1], 4096)):
        m.set_prefill_rows(rows)
        m.reset(1, 512)
        check(run_all(m, t, cut), ref, compute, "memory")


@both
def test_long_prompts_in_segments(compute):
    """Prompts long enough to be cut into segments that run beside each other, from the start and behind earlier tokens, one and several requests."""
    cfg = config([lightning(heads=2, dim=24, vdim=40, decay=[0.9995, 0.97], mlp=None), parallel(left(heads=2, kv_heads=1, window=30), right(32, 2, 2), mlp=None),
                  lightning(heads=1, dim=64, vdim=64, decay=[1.0], mlp=None)], width=64, vocab=50)
    W, m = build(cfg, compute)
    seqs = [tokens(n, 50, 70 + n) for n in (2300, 1090, 40)]
    refs = [orc.forward(cfg, W, t) for t in seqs]
    m.reset(1, 2304)
    for cut in ([2300], [130, 2170], [1300, 900, 1]):
        m.reset(1, 2304)
        got = run_all(m, seqs[0], cut)
        check(got, refs[0], compute, "segments")
    m.reset(3, 2304)
    got = m.extend([(b, t) for b, t in enumerate(seqs)], [list(range(len(t))) for t in seqs])
    check(got, np.concatenate(refs), compute, "segments")


@both
def test_convolution_across_portions(compute):
    """A convolution longer than the portions: its inputs come from several of them."""
    cfg = one_side(config([parallel(left(window=4), right(48, 3, 7), mlp=None)], width=64, vocab=50), "right")
    W, m = build(cfg, compute)
    t = tokens(40, 50, 17)
    ref = orc.forward(cfg, W, t)
    for cut in ([40], [1], [2], [3, 1, 4], [5, 2], [6, 1, 1, 9]):
        m.reset(1, 64)
        check(run_all(m, t, cut), ref, compute, "conv")


def test_first_tokens():
    """Positions 0, 1, 2 in every way of starting a sequence."""
    cfg = odd()
    for compute in ("float32", "bfloat16"):
        W, m = build(cfg, compute)
        t = tokens(3, cfg["vocab"], 14)
        ref = orc.forward(cfg, W, t)
        for cut in ([3], [1, 2], [2, 1], [1]):
            m.reset(1, 4)
            check(run_all(m, t, cut), ref, compute, "first")


def test_passes_of_a_loop_keep_their_own_state():
    cfg = config([parallel(), lightning()], loop=(0, 2, 3))
    W, m = build(cfg, "float32")
    assert {k.split(".")[0] for k in W if k[0] == "l"} == {"l0", "l1"}
    t = tokens(60, cfg["vocab"], 4)
    m.reset(1, 64)
    check(run_all(m, t, [9, 3, 1]), orc.forward(cfg, W, t), "float32", "loop")


# ---------------------------------------------------------------- generation: sampler, captured graph, stream
def greedy_margin(cfg, W, prompt, new):
    """For every generated id: the oracle's logit of the best id minus that of the generated one."""
    lg = orc.forward(cfg, W, list(prompt) + [int(x) for x in new[:-1]])[len(prompt) - 1:]
    return np.asarray([l.max() - l[i] for l, i in zip(lg, new)]), np.abs(lg).max()


@pytest.mark.parametrize("compute,slack", [("float32", 1e-4), ("bfloat16", 0.03)])
@pytest.mark.parametrize("shape", ["odd", "wide"])
def test_greedy_generation(shape, compute, slack):
    cfg = SHAPES[shape]()
    W, m = build(cfg, compute)
    prompts = [tokens(n, cfg["vocab"], 30 + n) for n in (3, 60, 1, 21)]
    gp = mas.GenerateParameters(max_tokens=40, temperature=0.0, repetition_penalty=1.0, repetition_context_size=0)
    first = m.generate_batch(prompts, gp)
    again = m.generate_batch(prompts, gp)                                       # the captured graph a second time, states from the start
    for p, a, b in zip(prompts, first, again):
        assert len(a) == 40 and np.array_equal(a, b)
        margin, scale = greedy_margin(cfg, W, p, a)
        assert observe(f"vamunex_greedy_margin_{compute}", float(margin.max() / scale), slack)
    # the loop has run its layers on every generated id: the rows stand behind them
    more = m.extend([(1, [int(first[1][0])])])
    ref = orc.forward(cfg, W, list(prompts[1]) + [int(x) for x in again[1]] + [int(first[1][0])])[-1:]
    check(more, ref, compute, "behind")
    # eager: the step function fed with the same ids chooses the same ones (float32: exactly)
    m.reset(1, 128)
    lg = m.extend([(0, prompts[1])])
    eager = []
    for i in range(40):
        eager.append(int(lg[0].argmax()))
        lg = m.extend([(0, [first[1][i]])])
    if compute == "float32":
        assert eager == first[1].tolist()
    else:
        assert np.mean(np.asarray(eager) == first[1]) > 0.9


def test_rows_that_stop_early():
    """A row that meets its stop id rests while the others go on: its state stays behind its last id, theirs are as without it."""
    cfg = odd()
    W, m = build(cfg, "float32")
    prompts = [tokens(n, cfg["vocab"], 60 + n) for n in (9, 4, 30)]
    gp = mas.GenerateParameters(max_tokens=24, temperature=0.0, repetition_penalty=1.0)
    free = m.generate_batch(prompts, gp)
    stop = int(free[1][7])
    cut = m.generate_batch(prompts, gp, stop_id=stop)
    for a, b in zip(free, cut):
        ids = a.tolist()
        assert b.tolist() == (ids[:ids.index(stop) + 1] if stop in ids else ids)
    ev = list(m.generate_stream_batch(prompts, gp))
    for b in range(3):
        assert [e.token for e in ev if isinstance(e, mas.TokenEvent) and e.row == b] == free[b].tolist()


def test_engine_calls_shared_with_the_other_models():
    """mis_lm_prefill / mis_lm_forward on the same handle type."""
    cfg = odd()
    W, m = build(cfg, "bfloat16")
    t = tokens(50, cfg["vocab"], 15)
    ref = orc.forward(cfg, W, t)
    lg = [m.prefill([t[:40], t[:7]], max_context=60)]
    for i in range(3):
        lg.append(m.forward([t[40 + i], t[7 + i]]))
    for i in range(4):
        check(lg[i][:1], ref[39 + i:40 + i], "bfloat16")
        check(lg[i][1:], ref[6 + i:7 + i], "bfloat16")
    m.forward([t[43], 0], active=[1, 0])                                        # row 1 stays where it was, its states too
    check(m.forward([t[44], t[10]])[1:], ref[10:11], "bfloat16")


def test_missing_and_wrong_tensors():
    cfg = odd()
    W = orc.random_weights(cfg, 1)
    m = mas.BlockLanguageModel(mas.BlockModelConfiguration.from_dict(cfg))
    for name, arr in (("l0.mix.left.q", W["l0.mix.left.q"][:-1]), ("l1.mix.left.q", W["l0.mix.left.q"]), ("l0.mix.q", W["l1.mix.q"]), ("l9.norm1", W["l0.norm1"]),
                      ("embed.norm", W["final.norm"]), ("l0.mix.right.ra", W["l0.mix.right.ra"][0])):
        with pytest.raises(mas.AudioGenerationError) as e:
            m.set_tensor(name, arr)
        assert e.value.case == "invalidInput"
    m.set_tensor("l2.norm2", W["l0.norm2"])                                     # (a norm of a feed-forward that is not there: nothing to keep)
    for k, v in W.items():
        if k != "l2.mix.right.lam":
            m.set_tensor(k, v)
    with pytest.raises(mas.AudioGenerationError) as e:
        m.finalize()
    assert "l2.mix.right.lam" in str(e.value)


# ---------------------------------------------------------------- directory, commands
def write_model(path, cfg, W):
    """config.json + model.safetensors (bfloat16)."""
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    head, blobs, at = {}, [], 0
    for k, v in W.items():
        b = (np.ascontiguousarray(v, np.float32).view(np.uint32) >> 16).astype("<u2").tobytes()
        head[k] = {"dtype": "BF16", "shape": list(v.shape), "data_offsets": [at, at + len(b)]}
        blobs.append(b); at += len(b)
    h = json.dumps(head).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(len(h).to_bytes(8, "little") + h + b"".join(blobs))


def test_directory_and_commands(tmp_path):
    cfg = odd()
    W = orc.random_weights(cfg, 21)
    d = str(tmp_path / "m")
    write_model(d, cfg, W)
    m = mas.load_model(d, compute="float32")
    t = tokens(30, cfg["vocab"], 22)
    ref = orc.forward(cfg, W, t)
    m.reset(1, 32)
    check(run_all(m, t), ref, "float32")
    ids = m.generate_batch([t[:5]], mas.GenerateParameters(max_tokens=6, temperature=0.0, repetition_penalty=1.0))[0]
    m.close()
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "lm_generate"), "--model", d, "--dtype", "float32", "--max-tokens", "6", "--prompt",
                        ",".join(str(x) for x in t[:5])], capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [int(x) for x in r.stdout.split()] == ids.tolist()
    out = tmp_path / "out"
    out.mkdir()
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": t[:20].tolist(), "want": [3, 19]}, {"id": "y", "tokens": t[:4].tolist(), "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "y", "tokens": [int(t[4])], "want": [0]}, {"id": "x", "tokens": [int(t[20])], "want": [0]}], "end": ["y"]},
             {"step": 2, "entries": [{"id": "x", "tokens": [int(t[21])], "want": []}], "end": []}]
    steps += [{"step": k, "entries": [{"id": "x", "tokens": [int(t[19 + k])], "want": [0]}], "end": ["x"] if k == 6 else []} for k in (3, 4, 5, 6)]
    steps += [{"step": 7, "entries": [{"id": "z", "tokens": t[:9].tolist(), "want": [8]}], "end": ["z"]}]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", d, "--dtype", "float32", "--out", str(out), "--max-tokens", "26"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == [f"done {k}" for k in range(8)]
    got = {i: np.fromfile(out / f"{i}.f32", "<f4").reshape(-1, cfg["vocab"]) for i in (0, 1, 3, 4, 5, 6, 7)}
    assert not (out / "2.f32").exists()
    check(got[0], ref[[3, 19]], "float32")
    check(got[1], ref[[4, 20]], "float32")
    for k in (3, 4, 5, 6):                                                      # the one that is left holds as much as both did
        check(got[k], ref[[19 + k]], "float32")
    check(got[7], ref[[8]], "float32")
