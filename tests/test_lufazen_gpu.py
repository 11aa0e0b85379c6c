"""The Lufazen design on the device against its plain restatement (lufazen_oracle.py): each mechanism alone at sizes the kernels pad,
tile and split differently, prompts cut in every way, mixed batches, slots and blocks used again, keys at block borders and far
away, long decoding, and generation through the framework's own entry points."""
import json
import os
import subprocess
import sys
from functools import partial
from pathlib import Path

import numpy as np
import pytest

import layered_helpers as H
import lufazen_models as LM
import lufazen_oracle as O
import potuzen_models as PM
from layered_helpers import TOL, build, cut, err, feed

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent
steady, greedy_oracle = partial(H.steady, O), partial(H.greedy_oracle, O)
ONE = {"f32": 1e-4, "bf16": 0.03}       # a single layer

SINGLE = {
    "latent-odd": (LM.latent(), 96), "latent-64": (LM.latent(heads=6, dim=64, rot=64, vdim=64, q_rank=96, kv_rank=64), 128),
    "latent-small-rotation": (LM.latent(dim=24, rot=2, vdim=32), 64), "latent-rot-16": (LM.latent(dim=16, rot=16, vdim=40, base=5e5), 64),
    "latent-rot-24": (LM.latent(dim=36, rot=24, vdim=16), 80),               # 16 does not divide it: turned by a launch of its own
    "latent-rot-80": (LM.latent(dim=20, rot=80, vdim=64), 64),               # no absorbed form for five steps of 16
    "latent-rot-128": (LM.latent(heads=2, dim=64, rot=128, vdim=128, kv_rank=128), 64),
    "latent-128+64": (LM.latent(heads=4, dim=128, rot=64, vdim=128, q_rank=192, kv_rank=512), 256),
    "latent-40+32-256": (LM.latent(heads=2, dim=40, rot=32, vdim=160), 64), "latent-100+60-200": (LM.latent(heads=2, dim=100, rot=60, vdim=200), 64),
    "latent-17-heads": (LM.latent(heads=17, dim=16, rot=16, vdim=8, kv_rank=256, scale=0.6), 96),
    "latent-kv-320": (LM.latent(heads=1, dim=8, rot=8, vdim=16, q_rank=5, kv_rank=320), 200),
    "latent-not-absorbable": (LM.latent(heads=2, dim=64, rot=32, vdim=64, kv_rank=576), 64),
    "latent-big-heads": (LM.latent(heads=2, dim=272, rot=64, vdim=264, scale=0.04), 64),
    "latent-negative-scale": (LM.latent(scale=-0.2), 64), "latent-no-scaling": (LM.latent(scaling=None, base=100.0), 64),
    "latent-scaling-to-the-last-pair": (LM.latent(scaling=(8.0, 4000, 700.0, 0.5), base=50.0), 64),
    "latent-steep-ramp": (LM.latent(scaling=(2.5, 100, 2.0, 1.9)), 64),
    "delta-odd": (LM.delta(), 96), "delta-64": (LM.delta(heads=4, kv_heads=4, dim=64, vdim=64, conv=3), 128),
    "delta-128": (LM.delta(heads=3, kv_heads=1, dim=128, vdim=128), 96), "delta-conv-1": (LM.delta(heads=3, kv_heads=3, dim=33, vdim=17, conv=1), 64),
    "delta-conv-2": (LM.delta(conv=2), 64), "delta-conv-6": (LM.delta(conv=6), 70), "delta-narrow": (LM.delta(heads=6, kv_heads=2, dim=6, vdim=5), 36),
    "delta-200": (LM.delta(heads=2, kv_heads=1, dim=200, vdim=70), 64), "delta-wide-values": (LM.delta(heads=2, kv_heads=2, dim=48, vdim=300), 64),
    "delta-300": (LM.delta(heads=2, kv_heads=1, dim=300, vdim=20), 64), "delta-limit": (LM.delta(limit=0.2), 64),
    "no-feed-forward": (LM.delta(ff=None), 96), "wide-row": (LM.delta(heads=1, kv_heads=1, dim=16, vdim=16, ff=16), 1100),
    "narrow": (LM.latent(heads=1, dim=4, rot=2, vdim=4, q_rank=3, kv_rank=2, ff=5), 12),
}


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("name", list(SINGLE))
def test_one_layer(gpu, tmp_path, name, precision):
    """A mechanism alone: a prompt in one piece, then the same in portions of 20 with the last tokens one by one, and in pairs."""
    layer, width = SINGLE[name]
    cfg = LM.config([layer], width=width, vocab=130)
    w = LM.weights(cfg, 7, a_rank=70 if name == "delta-64" else 7, g_rank=3 if name == "delta-128" else 11)
    g = np.random.default_rng(1)
    tok, want = steady(cfg, w, lambda: g.integers(0, 130, 149).tolist())
    layers = O.forward(cfg, w, tok, return_layers=True)[1]
    m = build(gpu, tmp_path, cfg, w, precision)
    m.set_debug(2)
    assert err(feed(m, 1, tok, [149]), want, precision) < ONE[precision]
    assert err(m.get_hidden(149), layers, precision) < ONE[precision]
    m.set_debug(0)
    assert err(feed(m, 2, tok, cut(129, 20) + [1] * 20), want, precision) < ONE[precision]
    assert err(feed(m, 3, tok, cut(149, 2)), want, precision) < ONE[precision]
    m.close()


@pytest.mark.parametrize("heads,dim,vdim", [(130, 20, 9), (130, 40, 24), (260, 40, 20), (256, 36, 72), (130, 72, 16), (260, 72, 16), (256, 72, 68), (130, 136, 16),
                                            (260, 136, 12), (256, 130, 66), (40, 130, 70)])
def test_delta_many_heads(gpu, tmp_path, heads, dim, vdim):
    """Every way the state scan splits columns and key channels over workgroups and waves."""
    cfg = LM.config([LM.delta(heads=heads, kv_heads=heads // 2, dim=dim, vdim=vdim, ff=None)], width=48, vocab=60)
    w = LM.weights(cfg, 13)
    g = np.random.default_rng(3)
    tok, want = steady(cfg, w, lambda: g.integers(0, 60, 45).tolist(), 0.05)
    m = build(gpu, tmp_path, cfg, w)
    for s, cuts in enumerate(([45], [7, 38], [33, 12])):
        assert err(feed(m, s, tok, cuts), want) < ONE["f32"]
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("decay_bias,a_log", [(30.0, (2.0, 6.0)), (-30.0, (0.1, 1.0)), (4.0, (6.0, 16.0)), (-5.0, (0.5, 2.0))])
def test_delta_decay_extremes(gpu, tmp_path, decay_bias, a_log, precision):
    """Decays close to 0 (a factor e^-60 per token and below: exponentials of the opposite sign would overflow inside a chunk) and
    close to 1 (nothing is forgotten but what is overwritten)."""
    cfg = LM.config([LM.delta(heads=4, kv_heads=4, dim=48, vdim=40)], width=96, vocab=90)
    w = LM.weights(cfg, 11, decay_bias=decay_bias, a_log=a_log)
    tok = np.random.default_rng(2).integers(0, 90, 200).tolist()
    want = O.forward(cfg, w, tok)
    m = build(gpu, tmp_path, cfg, w, precision)
    for cuts in ([200], cut(200, 37), [180] + [1] * 20):
        got = feed(m, len(cuts), tok, cuts)
        # (with everything forgotten a head's output is a multiple of v, whose norm flips its sign where q . k vanishes: the median position)
        e = np.sqrt(((got - want) ** 2).mean(axis=1)) / np.sqrt((want ** 2).mean())
        assert np.isfinite(got).all() and np.median(e) < (5e-6 if precision == "f32" else 0.03) and np.sort(e)[-10] < TOL[precision]
    m.close()


def test_delta_same_key_again_and_again(gpu, tmp_path):
    """One token repeated: all keys of a chunk are the same, step sizes near 1 — the triangular system at its worst, where a power series
    for its inverse would lose all digits."""
    cfg = LM.config([LM.delta(heads=3, kv_heads=3, dim=64, vdim=32, conv=1)], width=64, vocab=20)
    w = LM.weights(cfg, 17, decay_bias=-30.0)
    w["l0.mix.b"] = PM.bf16(w["l0.mix.b"] * 0 + 4.0 * np.sign(w["embed"][5])[None] / 64)
    tok = [5] * 70 + [6, 7] + [5] * 60
    want = O.forward(cfg, w, tok)
    m = build(gpu, tmp_path, cfg, w)
    for cuts in ([132], cut(132, 31), [100] + [1] * 32):
        assert err(feed(m, len(cuts), tok, cuts), want) < ONE["f32"]
    m.close()


def mixed_config():
    return LM.config([LM.latent(), LM.delta(), LM.latent(heads=2, dim=64, rot=32, vdim=48, kv_rank=40, base=300.0, ff=None), LM.latent(heads=5, dim=20, vdim=32, kv_from=0),
                      LM.delta(heads=2, kv_heads=2, dim=64, vdim=64, conv=3, ff=200), LM.latent(heads=1, dim=30, rot=32, vdim=48, kv_rank=40, base=300.0, kv_from=2),
                      LM.latent(kv_from=0, scale=0.3, ff=None), LM.delta(ff=None)], width=168, vocab=259, eps=2e-6)


@pytest.fixture(scope="module")
def stack():
    """One model with every mechanism, latents shared across layers in several ways, and its logits for four sequences."""
    cfg = mixed_config()
    w = LM.weights(cfg, 21)
    g = np.random.default_rng(5)
    both = [steady(cfg, w, lambda n=n: g.integers(0, 259, n).tolist(), 0.05) for n in (331, 70, 203, 6)]
    return cfg, w, [b[0] for b in both], [b[1] for b in both]


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("cuts", ["whole", "ones", "twos", "3", "16", "17", "31", "32", "33", "63", "64", "65", "128", "ragged", "tail"])
def test_portions(gpu, tmp_path, stack, cuts, precision):
    cfg, w, seqs, want = stack
    n = len(seqs[0])
    plan = dict(whole=[n], ones=[1] * n, twos=cut(n, 2), ragged=[2, 64, 3, 1, 1, 29, 128, 5, 16, 50, 32], tail=[n - 60] + [1] * 60).get(cuts) or cut(n, int(cuts))
    m = build(gpu, tmp_path, cfg, w, precision)
    assert err(feed(m, 3, seqs[0], plan), want[0], precision) < TOL[precision]
    m.close()


def test_cuts_and_company_do_not_show(gpu, tmp_path, stack):
    """fp32: the same positions from different cuts, slots and batches agree to rounding, far below their distance from the restatement's
    tolerance."""
    cfg, w, seqs, want = stack
    m = build(gpu, tmp_path, cfg, w)
    a = feed(m, 1, seqs[2], [203])
    b = feed(m, 2, seqs[2], cut(203, 45))
    m.seq_open(3)
    m.seq_open(4)
    toks, _ = m.forward_rows([4, 3], [seqs[0][:100], seqs[2][:150]], [0, 0], range(250))
    more, _ = m.forward_rows([3, 4], [seqs[2][150:], seqs[0][100:101]], [150, 100], range(53))
    assert err(b, a) < 2e-5 and err(np.concatenate([toks[100:], more]), a) < 2e-5
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
def test_long_prompts(gpu, tmp_path, precision):
    """Long portions from a zero and from a carried state; positions far beyond the rotation's original length."""
    cfg = LM.config([LM.delta(heads=2, kv_heads=1, dim=40, vdim=72), LM.latent(rot=32), LM.delta(heads=4, kv_heads=4, dim=70, vdim=32), LM.latent(rot=32, kv_from=1)], width=96, vocab=100)
    w = LM.weights(cfg, 31, decay_bias=-4.0)
    g = np.random.default_rng(3)
    tok, want = steady(cfg, w, lambda: g.integers(0, 100, 1200).tolist(), 0.08)
    m = build(gpu, tmp_path, cfg, w, precision, max_seq_len=1216, max_batch_tokens=1216)
    for cuts in ([1200], [600, 5, 400, 195], [513] + [1] * 7 + [680]):
        assert err(feed(m, len(cuts), tok, cuts), want, precision) < TOL[precision]
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
def test_mixed_batches_and_reuse(gpu, tmp_path, stack, precision):
    """Portions of some sequences beside single tokens of others, sequences left out of steps, slots and blocks given back and used
    again: every logit as if the sequence were alone.  The pool is exactly as large as the live sequences need."""
    cfg, w, seqs, want = stack
    m = build(gpu, tmp_path, cfg, w, precision, max_seqs=4, kv_num_blocks=sum(-(-len(s) // 64) for s in seqs))
    got, ref = H.mixed_run(m, seqs, want, [0, 1, 2, 3, 1, 3, 2, 0, 3, 1], 17)
    assert err(got, ref, precision) < TOL[precision]
    m.close()


def test_step_without_logits(gpu, tmp_path, stack):
    cfg, w, seqs, want = stack
    m = build(gpu, tmp_path, cfg, w)
    m.seq_open(1)
    lg, am = m.forward_rows([1], [seqs[1][:40]], [0], [])
    assert lg.shape == (0, 259) and am.size == 0
    assert err(feed(m, 1, seqs[1], [30]), want[1][40:]) < TOL["f32"]
    m.close()


# ---- single keys that stand out: far away, at block borders, the first tokens ----
def spotlight(cfg, w, A, B, score=25.0):
    """Queries of token B look for token A: the unrotated part of W_uq gets a term that adds `score` to that one score in every head."""
    w = dict(w)
    mx, eps = cfg["layers"][0]["mixer"], cfg["norm"]["eps"]
    n, d = mx["heads"], mx["dim"]
    h = {t: np.asarray(w["embed"][t], np.float64) for t in (A, B)}
    cq = O.rms_norm(w["l0.mix.dq"] @ h[B], w["l0.mix.dq.norm"], eps)
    k = (w["l0.mix.uk"] @ O.rms_norm((w["l0.mix.dkv"] @ h[A])[:mx["kv_rank"]], w["l0.mix.dkv.norm"], eps)).reshape(n, d)
    uq = np.array(w["l0.mix.uq"], np.float64).reshape(n, d + mx["rot_dim"], -1)
    for i in range(n):
        uq[i, :d] += np.outer(k[i] * (score / mx["scale"] / (k[i] @ k[i])), cq / (cq @ cq))
    w["l0.mix.uq"] = PM.bf16(uq.reshape(n * (d + mx["rot_dim"]), -1))
    return w


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("heads,dim,rot", [(17, 16, 16), (2, 48, 32)])
def test_far_key_among_hundreds(gpu, tmp_path, heads, dim, rot, precision):
    A, B, V = 77, 88, 90
    cfg = LM.config([LM.latent(heads=heads, dim=dim, rot=rot, vdim=16, q_rank=48, kv_rank=128, scale=0.3, ff=None)], width=128, vocab=V)
    w = spotlight(cfg, LM.weights(cfg, 43), A, B)
    m = build(gpu, tmp_path, cfg, w, precision)
    g = np.random.default_rng(8)
    for i, at in enumerate((0, 1, 5, 63, 64, 127, 128, 300, 575, 599)):
        tok = g.integers(0, A, 640)
        tok[at], tok[600], tok[639] = A, B, B
        tok = tok.tolist()
        want = O.forward(cfg, w, tok)
        gone = list(tok)
        gone[at] = 3
        assert err(O.forward(cfg, w, gone)[639:], want[639:]) > 0.3
        for cuts in ([590, 40] + [1] * 10, cut(640, 64), [601, 39]):
            got = feed(m, 10 * i + len(cuts), tok, cuts)
            assert err(got[[600, 639]], want[[600, 639]], precision) < ONE[precision], (at, cuts)
            m.seq_close(10 * i + len(cuts))
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
def test_rotated_scores_place_the_keys(gpu, tmp_path, precision):
    """Scores from the rotated part alone, and strong: the restatement with every position one off in the keys only is far away, and so is
    one without the context extension."""
    layer = LM.latent(heads=3, dim=8, rot=32, vdim=24, kv_rank=64, scale=0.4, ff=None)
    cfg = LM.config([layer], width=96, vocab=70)
    w = LM.weights(cfg, 47, rot_scale=2.5)
    w["l0.mix.uk"] = w["l0.mix.uk"] * 0
    tok = np.random.default_rng(9).integers(0, 70, 300).tolist()
    want = O.forward(cfg, w, tok)
    plain = dict(cfg, layers=[LM.latent(heads=3, dim=8, rot=32, vdim=24, kv_rank=64, scale=0.4, ff=None, scaling=None)])
    assert err(O.forward(plain, w, tok), want) > 0.3
    keep = O.latents
    try:
        O.latents = lambda h, m, mx, eps: (lambda c, k: (c, np.concatenate([k[:1], O.rotate(np.concatenate([(h @ m["dkv"].T)[:1, mx["kv_rank"]:], (h @ m["dkv"].T)[:, mx["kv_rank"]:]]), mx["rot"])[2:]])))(*keep(h, m, mx, eps))
        assert err(O.forward(cfg, w, tok), want) > 0.3
    finally:
        O.latents = keep
    m = build(gpu, tmp_path, cfg, w, precision)
    for s, cuts in enumerate(([300], [250] + [1] * 50, cut(300, 33))):
        assert err(feed(m, s, tok, cuts), want, precision) < (2e-4 if precision == "f32" else 0.2)
    m.close()


# ---- the framework's own entry points ----
def test_greedy_generation(gpu, tmp_path, stack):
    """Stepwise, fused on the device, and through the runner give the restatement's tokens (fp32)."""
    cfg, w, seqs, _ = stack
    prompt = seqs[1][:45]
    want, gap = greedy_oracle(cfg, w, prompt, 12)
    assert gap > 1e-3
    m = build(gpu, tmp_path, cfg, w)
    assert m.greedy(prompt, 12, seq_id=1) == want
    assert m.greedy_fused(prompt, 12, seq_id=2) == want
    r = gpu.HipModelRunner(m)
    s = gpu.Sequence(seq_id=9, token_ids=list(prompt))
    s.append_token(r.run([s], True)[0])
    for _ in range(11):
        s.append_token(r.run([s], False)[0])
    assert s.token_ids[len(prompt):] == want
    m.close()


def test_long_fused_decode_bf16(gpu, tmp_path, stack):
    """400 steps on the device for a batch of unequal sequences (captured passes) against the same steps one call at a time; the last
    logits against the restatement of what was generated."""
    cfg, w, seqs, _ = stack
    m = build(gpu, tmp_path, cfg, w, "bf16", max_seqs=3, kv_num_blocks=30)
    prompts, first = [seqs[0][:90], seqs[1][:7], seqs[2][:64]], []
    for i, p in enumerate(prompts):
        m.seq_open(i)
        first.append(int(m.forward_batch([i], [p], [0])[1][0]))
    out = m.decode_greedy([0, 1, 2], first, 400)
    again = []
    for i in range(3):
        m.seq_close(i)
        m.seq_open(10 + i)
        assert int(m.forward_batch([10 + i], [prompts[i]], [0])[1][0]) == first[i]
    tok = list(first)
    for s in range(400):
        _, am = m.forward_batch([10, 11, 12], [[t] for t in tok], [len(p) + s for p in prompts])
        tok = [int(t) for t in am]
        again.append(tok)
    assert np.array_equal(out, np.asarray(again))
    assert m.stats()["graph_replays"] > 700
    for i, p in enumerate(prompts):
        full = p + [first[i]] + out[:, i].tolist()
        want = O.forward(cfg, w, full)[-1]
        got, _ = m.forward_batch([10 + i], [[full[-1]]], [len(full) - 1])
        assert err(got, want[None]) < TOL["bf16"]
    m.close()


def test_runner_batches_evict_and_refill(gpu, tmp_path, stack):
    """More sequences than slots, and a pool smaller than all of them: the runner closes the least recently used one and prefills it
    again when it comes back."""
    cfg, w, seqs, _ = stack
    m = build(gpu, tmp_path, cfg, w, max_seqs=2, kv_num_blocks=7)
    r = gpu.HipModelRunner(m)
    want = {k: greedy_oracle(cfg, w, seqs[k][:n], 4) for k, n in ((0, 130), (1, 60), (2, 100))}
    assert min(v[1] for v in want.values()) > 1e-3
    live = {k: gpu.Sequence(seq_id=k, token_ids=list(seqs[k][:n])) for k, n in ((0, 130), (1, 60), (2, 100))}
    for k, s in live.items():
        s.append_token(r.run([s], True)[0])
    for _ in range(3):
        for pair in ([0, 1], [2]):
            for k, t in zip(pair, r.run([live[k] for k in pair], False)):
                live[k].append_token(t)
    assert m.stats()["evictions"] > 0
    for k, s in live.items():
        assert s.token_ids[-4:] == want[k][0]
    m.close()


def test_prompt_longer_than_a_call(gpu, tmp_path, stack):
    cfg, w, seqs, want = stack
    m = build(gpu, tmp_path, cfg, w, max_batch_tokens=100)
    s = gpu.Sequence(seq_id=1, token_ids=list(seqs[0]))
    toks, lg = gpu.HipModelRunner(m).run([s], True, return_logits=True)
    assert err(lg, want[0][-1:]) < TOL["f32"] and toks[0] == int(want[0][-1].argmax())
    m.close()


def test_sampling(gpu, tmp_path, stack):
    """The sampler on this model's capped logits: top_k = 1 is the argmax, in the runner and in the fused loop; a draw follows the
    distribution."""
    cfg, w, seqs, want = stack
    m = build(gpu, tmp_path, cfg, w, "bf16")
    prompt = seqs[1][:50]
    greedy = m.greedy(prompt, 6, seq_id=1)
    m.seq_reset(2)
    lg, am = m.forward_batch([2], [prompt], [0])
    assert np.abs(lg).max() <= cfg["logit_softcap"]
    assert m.sample([None], [0.4], top_k=1, repetition_penalty=1.0)[0] == greedy[0]
    p = np.exp(lg[0].astype(np.float64) - lg[0].max())
    p /= p.sum()
    u = 0.37
    got = int(m.sample([None], [u], repetition_penalty=1.0)[0])
    c = np.cumsum(p)
    assert c[got] >= u - 1e-4 and (got == 0 or c[got - 1] <= u + 1e-4)
    out = m.decode_sampled([2], [greedy[0]], 5, [list(prompt) + greedy[:1]], np.full((5, 1), 0.5), top_k=1, repetition_penalty=1.0)
    assert out[:, 0].tolist() == greedy[1:]
    m.close()


def test_command_line(gpu, tmp_path, stack):
    """examples/ask_greedy (the C consumer of the ABI) generates from a Lufazen folder."""
    exe = ROOT / "examples" / "ask_greedy"
    if not exe.exists():
        pytest.skip("examples/ask_greedy is not built")
    cfg, w, seqs, _ = stack
    PM.write(tmp_path, cfg, w)
    want, gap = greedy_oracle(cfg, w, seqs[3], 5)
    assert gap > 1e-3
    r = subprocess.run([str(exe), str(tmp_path), "5", *map(str, seqs[3])], capture_output=True, text=True, timeout=100, env=dict(os.environ, NVL_F32="1"))
    assert r.returncode == 0, r.stderr
    assert [int(t) for t in r.stdout.split()] == want


@pytest.mark.parametrize("dtype,precision", [("float32", "f32"), ("bfloat16", "bf16")])
def test_trace_run(gpu, tmp_path, stack, dtype, precision):
    cfg, w, seqs, want = stack
    PM.write(tmp_path / "m", cfg, w)
    (tmp_path / "o").mkdir()
    steps = [dict(step=0, entries=[dict(id="a", tokens=seqs[0][:100], want=[0, 99]), dict(id="b", tokens=seqs[3], want=[5, 2])], end=["b"]),
             dict(step=1, entries=[dict(id="a", tokens=seqs[0][100:101], want=[])], end=[]),
             dict(step=2, entries=[dict(id="c", tokens=seqs[1][:2], want=[1]), dict(id="a", tokens=seqs[0][101:140], want=[38])], end=["a", "c"])]
    r = subprocess.run([sys.executable, str(ROOT / "bin" / "trace_run"), "--model", str(tmp_path / "m"), "--dtype", dtype, "--out", str(tmp_path / "o"),
                        "--max-tokens", "256"], input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"]
    read = lambda n: np.fromfile(tmp_path / "o" / f"{n}.f32", "<f4").reshape(-1, 259)
    assert err(read(0), np.stack([want[0][0], want[0][99], want[3][5], want[3][2]]), precision) < TOL[precision]
    assert not (tmp_path / "o" / "1.f32").exists()
    assert err(read(2), np.stack([want[1][1], want[0][139]]), precision) < TOL[precision]
