"""Rugunex on the device against oracle/rugunex.py: each mechanism alone (the other branches' layer scales are zero, or the residual stream is read
behind every layer), prompts against token-by-token decoding, portions, batches, rows used again, window edges with scores that stand out, and
generation through the engine's own loop (captured graph, sampler) - in bfloat16 and in the 32-bit mode."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import mlx_audio_swift_amd as mas
from oracle import rugunex as orc
from rugunex_util import config, huge, many, middle, mixer, no_branch, odd, rel_rms, row_rel_rms, standout, wide
from gpu_util import observe

pytestmark = pytest.mark.gpu
# relative rms error of the logits (mean taken off the reference); rows: of the worst row
TOL = {"float32": 5e-6, "bfloat16": 1.2e-2}
SHAPES = {"odd": odd, "wide": wide, "middle": middle, "many": many, "huge": huge}
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


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


def check(got, ref, compute, kind="logits"):
    assert np.isfinite(got).all()
    assert observe(f"{kind}_{compute}", row_rel_rms(got, ref), TOL[compute])


# ---------------------------------------------------------------- mechanisms alone
@pytest.mark.parametrize("compute", ["float32", "bfloat16"])
def test_embedding_norm_and_capped_head(compute):
    cfg = config(width=100, vocab=130, logit_scale=3.0, logit_softcap=4.0)
    W = no_branch(no_branch(orc.random_weights(cfg, 1), "ls1"), "ls2")
    m = mas.BlockLanguageModel.from_weights(cfg, W, compute=compute)
    t = tokens(70, 130)
    m.reset(1, 80)
    got, res = m.extend([(0, t)], [list(range(70))], return_residual=True)
    ref, layers = orc.forward(cfg, W, t, return_layers=True)
    assert np.abs(ref).max() > 3.9                                              # the cap bends these logits
    assert np.abs(res[0] - layers[0]).max() < 1e-5 * np.abs(layers[0]).max()    # float32 residual in both modes
    check(got, ref, compute)


@pytest.mark.parametrize("compute", ["float32", "bfloat16"])
@pytest.mark.parametrize("branch", ["ls1", "ls2"])
@pytest.mark.parametrize("shape", list(SHAPES))
def test_one_branch_alone(shape, branch, compute):
    """ls1 = 0: feed-forward only; ls2 = 0: latent attention only.  Compared in the residual stream behind every layer."""
    cfg = SHAPES[shape]()
    W = no_branch(orc.random_weights(cfg, 2), branch)
    m = mas.BlockLanguageModel.from_weights(cfg, W, compute=compute)
    t = tokens(90, cfg["vocab"], 3)
    m.reset(1, 96)
    _, res = m.extend([(0, t)], [[]], return_residual=True)
    _, layers = orc.forward(cfg, W, t, return_layers=True)
    for a, b in zip(res, layers):
        check(a, b, compute, "residual")


def test_layers_that_share_weights_keep_their_own_cache():
    cfg = config(layers=[dict(mixer=mixer()), dict(mixer=mixer(), weights_of=0), dict(mixer=mixer(), weights_of=0)])
    W, m = build(cfg, "float32")
    assert {k.split(".")[0] for k in W if k[0] == "l"} == {"l0"}
    t = tokens(40, cfg["vocab"], 4)
    m.reset(1, 48)
    check(run_all(m, t, [9, 3, 1]), orc.forward(cfg, W, t), "float32")


# ---------------------------------------------------------------- whole prompts, portions, decoding
@pytest.mark.parametrize("compute", ["float32", "bfloat16"])
@pytest.mark.parametrize("shape", list(SHAPES))
def test_prompt_portions_and_decoding(shape, compute):
    """One pass, passes of a few rows, portions down to two tokens, and token by token - all against the oracle."""
    cfg = SHAPES[shape]()
    W, m = build(cfg, compute)
    n = 260 if shape == "wide" else 190
    t = tokens(n, cfg["vocab"], 5)
    ref = orc.forward(cfg, W, t)
    for cut, rows in (([n], 4096), ([n], 50), ([n], 64), ([64, 33, 65, 2], 4096), ([n - 40, 1], 4096), ([1], 4096)):
        m.set_prefill_rows(rows)
        m.reset(1, n)
        got = run_all(m, t, cut)
        assert observe(f"cut{cut[0]}_{rows}_{compute}", row_rel_rms(got, ref), TOL[compute]), (cut, rows)


@pytest.mark.parametrize("compute", ["float32", "bfloat16"])
def test_long_decoding(compute):
    """Many windows past the prompt, in shares of keys (wide) as well."""
    cfg = config(width=128, vocab=97, ff=64, layers=[dict(mixer=mixer(heads=2, dim=16, rot_dim=8, vdim=16, kv_rank=32, window=100))] * 2)
    W, m = build(cfg, compute)
    t = tokens(700, 97, 6)
    m.reset(1, 700)
    check(run_all(m, t, [5, 1]), orc.forward(cfg, W, t), compute)


@pytest.mark.parametrize("compute", ["float32", "bfloat16"])
@pytest.mark.parametrize("shape", ["odd", "wide"])
def test_batch_of_unequal_requests(shape, compute):
    """Prompts of different lengths in one batch, decoded together while the short ones end: every row as if it were alone."""
    cfg = SHAPES[shape]()
    W, m = build(cfg, compute)
    lens, extra = [1, 77, 2, 160, 33], [30, 5, 0, 12, 30]
    seqs = [tokens(a + b, cfg["vocab"], 20 + i) for i, (a, b) in enumerate(zip(lens, extra))]
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
        o = np.concatenate(out[b])
        check(o, orc.forward(cfg, W, s), compute)
        m2_rows = m                                                             # the same request alone
    m2_rows.reset(1, 200)
    alone = run_all(m2_rows, seqs[3], [lens[3], 1])
    assert observe(f"alone_{compute}", row_rel_rms(np.concatenate(out[3]), alone), TOL[compute])


@pytest.mark.parametrize("compute", ["float32", "bfloat16"])
def test_rows_used_again(compute):
    """A reset gives the rows back: nothing of an earlier, longer request shows in what comes after it, at the same and at other batch sizes."""
    cfg = odd()
    W, m = build(cfg, compute)
    a, b = tokens(120, cfg["vocab"], 7), tokens(31, cfg["vocab"], 8)
    ref = orc.forward(cfg, W, b)
    m.reset(2, 128)
    m.extend([(0, a), (1, a[::-1])], [[], []])
    for batch, row in ((2, 1), (2, 0), (1, 0), (3, 2), (2, 1)):
        m.reset(batch, 128)
        check(run_all(m, b, [20, 1], row=row), ref, compute)


@pytest.mark.parametrize("compute", ["float32", "bfloat16"])
def test_more_rows_than_one_tile(compute):
    cfg = config(width=96, vocab=64, ff=64, layers=[dict(mixer=mixer(heads=2, dim=16, rot_dim=4, vdim=8, kv_rank=24, window=6))])
    W, m = build(cfg, compute)
    seqs = [tokens(3 + b % 5 + 4, 64, b) for b in range(64)]
    m.reset(64, 16)
    m.extend([(b, s[:-4]) for b, s in enumerate(seqs)], [[] for _ in seqs])
    outs = [m.extend([(b, s[len(s) - 4 + k:len(s) - 4 + k + 1]) for b, s in enumerate(seqs)]) for k in range(4)]
    for b, s in enumerate(seqs):
        check(np.stack([o[b] for o in outs]), orc.forward(cfg, W, s)[-4:], compute)


# ---------------------------------------------------------------- window edges that show
@pytest.mark.parametrize("compute", ["float32", "bfloat16"])
@pytest.mark.parametrize("window", [1, 2, 31, 32, 33, 64, 65, 150])
def test_window_edge(window, compute):
    """A query whose score with ONE key stands out: the key just inside the window decides the output, just outside it must not - wherever the edge
    falls in a tile of keys, a portion, a pass, and in decoding."""
    cfg = config(width=256, vocab=80, ff=64, layers=[dict(mixer=mixer(heads=4, dim=32, rot_dim=8, vdim=32, kv_rank=64, window=window), mlp=None)])
    W = standout(cfg, orc.random_weights(cfg, 9), 0, key_token=70, query_token=71, gain=14.0)
    m = mas.BlockLanguageModel.from_weights(cfg, W, compute=compute)
    base = tokens(230, 70, 10)
    refs = {}
    for off in (window - 1, window):                                            # distance from the query to the key: inside, outside
        if off == 0:
            continue                                                            # (the query itself)
        for q in (window + 3, 190):
            t = base.copy()
            t[q], t[q - off] = 71, 70
            plain = t.copy(); plain[q - off] = base[q - off]
            ref = orc.forward(cfg, W, t[:q + 1])
            refs[off, q] = np.abs(ref[q] - orc.forward(cfg, W, plain[:q + 1])[q]).max()
            for cut, rows in (([q + 1], 4096), ([q + 1], 37), ([q, 1], 4096), ([max(q - off, 1), 2], 4096)):
                m.set_prefill_rows(rows)
                m.reset(1, 256)
                check(run_all(m, t[:q + 1], cut)[q:], ref[q:], compute, "edge")
    for (off, q), moved in refs.items():                                        # the oracle: seen inside, not at all outside
        assert moved > 1.0 if off < window else moved < 1e-9


@pytest.mark.parametrize("compute", ["float32", "bfloat16"])
def test_far_key_among_hundreds(compute):
    """No window: one key far back stands out, in a prompt and in decoding (key shares meet over 400 keys)."""
    cfg = config(width=256, vocab=80, ff=64, layers=[dict(mixer=mixer(heads=4, dim=64, rot_dim=8, vdim=32, kv_rank=96, window=None), mlp=None)])
    W = standout(cfg, orc.random_weights(cfg, 12), 0, key_token=70, query_token=71, gain=16.0)
    m = mas.BlockLanguageModel.from_weights(cfg, W, compute=compute)
    for key in (0, 1, 31, 32, 255, 398):
        t = tokens(400, 70, 13)
        t[key], t[399] = 70, 71
        ref = orc.forward(cfg, W, t)
        for cut in ([400], [399, 1], [70, 329, 1]):
            m.reset(1, 400)
            check(run_all(m, t, cut)[399:], ref[399:], compute, "far")


def test_first_tokens():
    """Positions 0, 1, 2 in every way of starting a sequence."""
    cfg = odd()
    for compute in ("float32", "bfloat16"):
        W, m = build(cfg, compute)
        t = tokens(3, cfg["vocab"], 14)
        ref = orc.forward(cfg, W, t)
        for cut in ([3], [1, 2], [2, 1], [1]):
            m.reset(1, 4)
            check(run_all(m, t, cut), ref, compute)


# ---------------------------------------------------------------- generation: sampler, captured graph, stream
def greedy_margin(cfg, W, prompt, new):
    """The oracle's continuation check: for every generated id, logit of the best id minus logit of the generated one."""
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
    again = m.generate_batch(prompts, gp)                                       # the captured graph a second time
    for p, a, b in zip(prompts, first, again):
        assert len(a) == 40 and np.array_equal(a, b)
        margin, scale = greedy_margin(cfg, W, p, a)
        assert observe(f"greedy_margin_{compute}", float(margin.max() / scale), slack)
    # the loop has run its layers on every generated id: the rows stand behind them
    more = m.extend([(1, [int(first[1][0])])])
    ref = orc.forward(cfg, W, list(prompts[1]) + [int(x) for x in again[1]] + [int(first[1][0])])[-1:]
    check(more, ref, compute)
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


def test_generation_options():
    cfg = odd()
    W, m = build(cfg, "bfloat16")
    prompts = [tokens(n, cfg["vocab"], 40 + n) for n in (4, 9)]
    greedy = m.generate_batch(prompts, mas.GenerateParameters(max_tokens=12, temperature=0.0, repetition_penalty=1.0))
    stop = int(greedy[0][5])
    k = greedy[0].tolist().index(stop) + 1
    cut = m.generate_batch(prompts, mas.GenerateParameters(max_tokens=12, temperature=0.0, repetition_penalty=1.0), stop_id=stop)
    assert cut[0].tolist() == greedy[0][:k].tolist()
    # a penalty on everything seen keeps greedy from repeating an id
    pen = m.generate_batch(prompts, mas.GenerateParameters(max_tokens=12, temperature=0.0, repetition_penalty=1e6, repetition_context_size=64))
    assert all(len(set(p.tolist())) == 12 for p in pen)
    # sampling: the same seed gives the same ids, rows keep theirs whatever the slicing, another seed differs
    gp = mas.GenerateParameters(max_tokens=24, temperature=1.0, top_p=0.95, repetition_penalty=1.0, seed=5)
    a = m.generate_batch(prompts, gp)
    assert all(np.array_equal(x, y) for x, y in zip(a, m.generate_batch(prompts, gp)))
    from dataclasses import replace
    assert not np.array_equal(a[0], m.generate_batch(prompts, replace(gp, seed=6))[0])
    alone = m.generate_batch(prompts[1:], replace(gp, row_offset=1))[0]
    assert np.mean(alone == a[1]) > 0.5                                         # (equal up to a draw on the edge of rounding)
    ev = list(m.generate_stream_batch(prompts, gp))
    for b in range(2):
        assert [e.token for e in ev if isinstance(e, mas.TokenEvent) and e.row == b] == a[b].tolist()
    info = [e for e in ev if isinstance(e, mas.InfoEvent)]
    assert [i.info.prompt_token_count for i in info] == [4, 9] and all(i.info.generation_token_count == 24 for i in info)


def test_engine_calls_shared_with_the_other_models():
    """mis_lm_prefill / mis_lm_forward on the same handle type, and the errors of the step function."""
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
    m.forward([t[43], 0], active=[1, 0])                                        # row 1 stays where it was
    check(m.forward([t[44], t[10]])[1:], ref[10:11], "bfloat16")
    m.reset(2, 64)
    for bad in ([(2, [1])], [(0, [1]), (0, [2])], [(0, [cfg["vocab"]])], [(0, [-1])], [(0, [1] * 65)]):
        with pytest.raises(mas.AudioGenerationError) as e:
            m.extend(bad)
        assert e.value.case == "invalidInput"
    with pytest.raises(mas.AudioGenerationError):
        m.set_tensor("embed", W["embed"])                                       # finalized


def test_missing_and_wrong_tensors():
    cfg = odd()
    W = orc.random_weights(cfg, 1)
    m = mas.BlockLanguageModel(mas.BlockModelConfiguration.from_dict(cfg))
    for name, arr in (("l0.mix.q", W["l0.mix.q"][:-1]), ("l2.norm1", W["l0.norm1"]), ("l0.mix.gate", W["l0.norm1"]), ("l9.norm1", W["l0.norm1"])):
        with pytest.raises(mas.AudioGenerationError) as e:
            m.set_tensor(name, arr)
        assert e.value.case == "invalidInput"
    for k, v in W.items():
        if k != "l3.mix.uv":
            m.set_tensor(k, v)
    with pytest.raises(mas.AudioGenerationError) as e:
        m.finalize()
    assert "l3.mix.uv" in str(e.value)


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
             {"step": 2, "entries": [{"id": "x", "tokens": [int(t[21])], "want": []}], "end": ["x"]},
             {"step": 3, "entries": [{"id": "z", "tokens": t[:9].tolist(), "want": [8]}], "end": ["z"]}]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", d, "--dtype", "float32", "--out", str(out), "--max-tokens", "40"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2", "done 3"]
    got = {i: np.fromfile(out / f"{i}.f32", "<f4").reshape(-1, cfg["vocab"]) for i in (0, 1, 3)}
    assert not (out / "2.f32").exists()
    check(got[0], ref[[3, 19]], "float32")
    check(got[1], ref[[4, 20]], "float32")
    check(got[3], ref[[8]], "float32")
