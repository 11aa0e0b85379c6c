"""The Bolinex design on the device against its plain restatement (bolinex_oracle.py): each mechanism alone at sizes the kernels pad,
tile and split differently, prompts cut in every way, mixed batches, slots and blocks used again, keys far away, at block borders and
at window edges, long decoding, and generation through the framework's own entry points."""
import json
import os
import subprocess
import sys
from functools import partial
from pathlib import Path

import numpy as np
import pytest

import bolinex_models as BM
import bolinex_oracle as O
import layered_helpers as H
import potuzen_models as PM
from layered_helpers import TOL, build, cut, err, feed

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent
greedy_oracle = partial(H.greedy_oracle, O)
ONE = {"f32": 1e-4, "bf16": 0.03}       # a single layer
att, moe = BM.attention, BM.moe

SINGLE = {      # layer, width, side
    "odd": (att(), 96, 20), "no-window": (att(window=None), 96, 20), "window-1": (att(window=1), 64, 20), "window-63": (att(window=63), 64, 20),
    "window-64": (att(window=64), 64, 20), "window-65": (att(window=65), 64, 20), "no-cap": (att(cap=None), 64, 20), "tight-cap": (att(cap=0.7, scale=0.6), 64, 20),
    "negative-scale": (att(scale=-0.3), 64, 20), "wide-cap": (att(cap=59.0, scale=9.0), 64, 20), "wider-cap": (att(cap=200.0, scale=9.0), 64, 20),
    "no-cap-long-table": (att(cap=None, window=None, heads=24, kv_heads=1, dim=64, vdim=64), 64, 20), "one-head-each": (att(heads=3, kv_heads=3), 96, 20), "one-kv-head": (att(heads=5, kv_heads=1), 96, 20),
    "group-17": (att(heads=34, kv_heads=2, dim=16, vdim=8, window=100), 96, 20), "group-70": (att(heads=70, kv_heads=1, dim=12, vdim=5), 64, 20),
    "32-32": (att(dim=32, vdim=32), 64, 20), "64-64": (att(heads=4, kv_heads=1, dim=64, vdim=64, window=None), 128, 64), "128-128": (att(heads=4, kv_heads=2, dim=128, vdim=128), 128, 20),
    "20-160": (att(heads=2, kv_heads=1, dim=20, vdim=160), 64, 20), "200-40": (att(heads=2, kv_heads=2, dim=200, vdim=40), 64, 20), "150-100": (att(heads=2, kv_heads=1, dim=150, vdim=100), 64, 20),
    "256-256": (att(heads=4, kv_heads=2, dim=250, vdim=256, scale=0.06), 96, 20), "big-heads": (att(heads=2, kv_heads=1, dim=272, vdim=264, scale=0.05), 64, 20),
    "narrow": (att(heads=1, kv_heads=1, dim=4, vdim=4, mlp=BM.dense(5)), 12, 3), "wide-row": (att(heads=2, kv_heads=1, mlp=BM.dense(16)), 1100, 20),
    "no-feed-forward": (att(mlp=None), 96, 20), "dense-200": (att(mlp=BM.dense(200)), 70, 100), "side-5": (att(mlp=None), 64, 5), "side-300": (att(mlp=None), 64, 300), "no-side": (att(mlp=moe()), 64, None),
    "shared-1100": (att(mlp=moe(4, 2, None, 24, 1100)), 64, 20),
    "experts": (att(mlp=moe()), 96, 20), "experts-5-of-one-group": (att(mlp=moe(5, 2, None, 24, None)), 64, 20), "one-expert": (att(mlp=moe(1, 1, None, 24, 30)), 64, 20),
    "experts-40": (att(mlp=moe(40, 6, (8, 3), 16, 8)), 64, 20), "experts-72": (att(mlp=moe(72, 5, (9, 4), 12, None)), 64, 20), "groups-of-one": (att(mlp=moe(6, 2, (6, 3), 24)), 64, 20),
    "all-of-the-kept": (att(mlp=moe(8, 4, (4, 2), 24)), 64, 20), "every-expert": (att(mlp=moe(6, 6, (3, 3), 24)), 64, 20), "wide-experts": (att(mlp=moe(6, 2, (2, 1), 200, 136)), 256, 20),
}


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("name", list(SINGLE))
def test_one_layer(gpu, tmp_path, name, precision):
    """A mechanism alone: a prompt in one piece, then the same in portions of 20 with the last tokens one by one, and in pairs."""
    layer, width, side = SINGLE[name]
    cfg = BM.config([layer], width=width, vocab=130, side=side, positions=160)
    w = BM.weights(cfg, 7)
    tok, want, layers = BM.clear_tokens(cfg, w, 149, 1)
    m = build(gpu, tmp_path, cfg, w, precision)
    m.set_debug(2)
    assert err(feed(m, 1, tok, [149]), want, precision) < ONE[precision]
    assert err(m.get_hidden(149), layers, precision) < ONE[precision]
    m.set_debug(0)
    assert err(feed(m, 2, tok, cut(129, 20) + [1] * 20), want, precision) < ONE[precision]
    assert err(feed(m, 3, tok, cut(149, 2)), want, precision) < ONE[precision]
    m.close()


def mixed_config():
    return BM.config([att(v_mix=False), att(mlp=moe()), att(heads=4, kv_heads=2, dim=64, vdim=24, window=None, cap=None, mlp=None), att(heads=2, kv_heads=2, dim=20, window=130, mlp=moe(8, 2, None, 72, None)),
                      att(heads=12, kv_heads=2, dim=16, window=64, scale=0.5, cap=4.0, v_mix=False, mlp=BM.dense(200)), att(heads=2, kv_heads=2, dim=100, window=33, mlp=moe(20, 4, (5, 3), 16, 100))],
                     width=168, vocab=259, eps=2e-6, side=28, positions=520)


@pytest.fixture(scope="module")
def stack():
    """One model with every mechanism, values mixed across layers that are not neighbours, and its logits for four sequences."""
    cfg = mixed_config()
    w = BM.weights(cfg, 21)
    both = [BM.clear_tokens(cfg, w, n, 5 + n) for n in (331, 70, 203, 6)]
    return cfg, w, [b[0] for b in both], [b[1] for b in both]


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("cuts", ["whole", "ones", "twos", "3", "10", "16", "17", "31", "32", "33", "63", "64", "65", "128", "ragged", "tail"])
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
def test_mixed_batches_and_reuse(gpu, tmp_path, stack, precision):
    """Portions of some sequences beside single tokens of others, sequences left out of steps, slots and blocks given back and used
    again: every logit as if the sequence were alone.  The pool is exactly as large as the live sequences need."""
    cfg, w, seqs, want = stack
    m = build(gpu, tmp_path, cfg, w, precision, max_seqs=4, kv_num_blocks=sum(-(-len(s) // 64) for s in seqs))
    got, ref = H.mixed_run(m, seqs, want, [0, 1, 2, 3, 1, 3, 2, 0, 3, 1], 17)
    assert err(got, ref, precision) < TOL[precision]
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
def test_windows_give_blocks_back(gpu, tmp_path, precision):
    """Windows in every layer: one long sequence runs in a pool of a few blocks, in portions and decoding, over blocks used again."""
    cfg = BM.config([att(window=70), att(window=20, mlp=moe(6, 2, (2, 1), 16, 8))], width=80, vocab=90, positions=460)
    w = BM.weights(cfg, 9)
    tok, want, _ = BM.clear_tokens(cfg, w, 450, 2)
    m = build(gpu, tmp_path, cfg, w, precision, max_seqs=2, kv_num_blocks=4)
    for s, cuts in enumerate((cut(450, 50), [64] * 3 + [1] * 258, cut(450, 17))):
        assert err(feed(m, s, tok, cuts), want, precision) < TOL[precision]
        m.seq_close(s)
    m.close()


def test_step_without_logits(gpu, tmp_path, stack):
    cfg, w, seqs, want = stack
    m = build(gpu, tmp_path, cfg, w)
    m.seq_open(1)
    lg, am = m.forward_rows([1], [seqs[1][:40]], [0], [])
    assert lg.shape == (0, 259) and am.size == 0
    assert err(feed(m, 1, seqs[1], [30]), want[1][40:]) < TOL["f32"]
    m.close()


# ---- single keys that stand out: far away, at block borders, at window edges, the first tokens ----
def spotlight(cfg, w, A, B, score=24.0):
    """Queries of token B look for token A in every head of layer 0, wherever the two stand: their embeddings get a direction of their
    own, which W_q and W_k turn into one pair of vectors that scores `score`."""
    w = dict(w)
    mx, W = cfg["layers"][0]["mixer"], cfg["width"]
    g = np.random.default_rng(99)
    u, v = np.linalg.qr(g.standard_normal((W, 2)))[0].T
    u, v = (x - x.mean() for x in (u, v))                                   # (layer norm takes the mean off)
    w["embed"], w["pos"] = np.array(w["embed"]), PM.bf16(0.1 * w["pos"])
    w["embed"][A], w["embed"][B] = PM.bf16(40 * u), PM.bf16(40 * v)
    h = {t: O.layer_norm(w["embed"][t].astype(np.float64), w["l0.norm1"], w["l0.norm1.b"], cfg["norm"]["eps"]) for t in (A, B)}
    k = g.standard_normal((mx["kv_heads"], mx["dim"]))
    q = np.repeat(k, mx["heads"] // mx["kv_heads"], axis=0)
    q = q * (score / mx["scale"] / (q * q).sum(axis=1, keepdims=True))
    w["l0.mix.k"] = PM.bf16(0.2 * w["l0.mix.k"] + np.outer(k.reshape(-1), h[A] / (h[A] @ h[A])))
    w["l0.mix.q"] = PM.bf16(0.2 * w["l0.mix.q"] + np.outer(q.reshape(-1), h[B] / (h[B] @ h[B])))
    w["l0.mix.o"] = PM.bf16(6.0 * w["l0.mix.o"])                            # (the residual at B is large: what attention brings should show)
    return w


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(17, 1, 16, 16), (4, 2, 72, 40)])
def test_far_key_among_hundreds(gpu, tmp_path, heads, kv_heads, dim, vdim, precision):
    A, B, V = 77, 88, 90
    cfg = BM.config([att(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, window=None, scale=0.3, cap=40.0, mlp=None)], width=128, vocab=V, side=8, positions=640)
    w = spotlight(cfg, BM.weights(cfg, 43, r1=(0.3, 1.2), r2=(0.05, 0.3)), A, B)
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
@pytest.mark.parametrize("window", [1, 2, 31, 64, 65, 100, 192])
def test_window_edges(gpu, tmp_path, window, precision):
    """A key just inside and one just outside the window of a query, at block borders and between them, in prompts and in decoding: what is
    outside leaves no trace, what is inside decides the row."""
    A, B, V = 77, 88, 90
    cfg = BM.config([att(heads=4, kv_heads=2, dim=32, vdim=32, window=window, scale=0.3, cap=40.0, mlp=None)], width=96, vocab=V, side=8, positions=420)
    w = spotlight(cfg, BM.weights(cfg, 44, r1=(0.3, 1.2), r2=(0.05, 0.3)), A, B)
    m = build(gpu, tmp_path, cfg, w, precision)
    g = np.random.default_rng(9)
    sid = 0
    for q in (200, 255, 256, 301, 319):
        base = g.integers(0, A, 320)
        base[q] = B
        rows = {}
        for name, back in (("in", window - 1), ("out", window)):
            tok = base.copy()
            if back > 0:
                tok[q - back] = A
            tok = tok.tolist()
            want = O.forward(cfg, w, tok)
            for cuts in ([320], [q] + [1] * (320 - q), [q - 20, 21, 319 - q] if q < 319 else cut(320, 2)):
                got = feed(m, sid, tok, cuts)
                assert err(got[[q]], want[[q]], precision) < ONE[precision], (q, name, cuts)
                m.seq_close(sid)
                sid += 1
            rows[name] = want[q]
        plain = O.forward(cfg, w, base.tolist())[q]
        assert np.array_equal(rows["out"], plain) or np.allclose(rows["out"], plain, atol=1e-12)
        assert window == 1 or err(rows["in"][None], plain[None]) > 0.3
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
def test_distance_bias_places_the_keys(gpu, tmp_path, precision):
    """Scores from the bias alone, and strong: the restatement with every distance one off, or with the bias under the cap, is far away."""
    cfg = BM.config([att(heads=3, kv_heads=1, dim=8, vdim=24, window=None, scale=0.4, cap=0.5, mlp=None)], width=96, vocab=70, side=4, positions=300)
    w = BM.weights(cfg, 47, r1=(1.5, 4.0), r2=(0.5, 3.0))
    tok = np.random.default_rng(9).integers(0, 70, 300).tolist()
    want = O.forward(cfg, w, tok)
    keep = O.distance_bias
    try:
        O.distance_bias = lambda r1, r2, back: keep(r1, r2, np.maximum(back - 1, 0))
        assert err(O.forward(cfg, w, tok), want) > 0.1
        O.distance_bias = lambda r1, r2, back: 0.5 * np.tanh(keep(r1, r2, back) / 0.5)
        assert err(O.forward(cfg, w, tok), want) > 0.1
    finally:
        O.distance_bias = keep
    m = build(gpu, tmp_path, cfg, w, precision)
    for s, cuts in enumerate(([300], [250] + [1] * 50, cut(300, 33))):
        assert err(feed(m, s, tok, cuts), want, precision) < ONE[precision]
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("r1,r2", [((-1.5, -0.5), (0.1, 0.4)), ((0.0, 0.0), (0.0, 0.0)), ((20.0, 40.0), (1.0, 3.0))])
def test_distance_bias_of_any_sign_and_size(gpu, tmp_path, r1, r2, precision):
    """Biases that raise far scores (a running maximum is needed), that are zero, and that bury everything but the nearest keys."""
    cfg = BM.config([att(heads=4, kv_heads=2, dim=32, vdim=32, window=None, mlp=None)], width=64, vocab=70, side=4, positions=300)
    w = BM.weights(cfg, 48, r1=r1, r2=r2)
    tok = np.random.default_rng(10).integers(0, 70, 300).tolist()
    want = O.forward(cfg, w, tok)
    m = build(gpu, tmp_path, cfg, w, precision)
    for s, cuts in enumerate(([300], [250] + [1] * 50, cut(300, 33))):
        assert err(feed(m, s, tok, cuts), want, precision) < ONE[precision]
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
def test_learned_positions_reach_their_end(gpu, tmp_path, precision):
    """As many tokens as there are positions, decoded to the last one; one more is refused."""
    cfg = BM.config([att(mlp=None)], width=64, vocab=60, side=4, positions=75)
    w = BM.weights(cfg, 4)
    tok, want, _ = BM.clear_tokens(cfg, w, 75, 3)
    m = build(gpu, tmp_path, cfg, w, precision)
    assert err(feed(m, 1, tok, [60] + [1] * 15), want, precision) < ONE[precision]
    with pytest.raises(gpu.NvlError):
        m.forward_batch([1], [[3]], [75])
    m.close()


@pytest.mark.parametrize("rows", [64, 65, 100, 300])
def test_expert_forms_agree(gpu, tmp_path, rows):
    """The masked form (up to 64 rows a call) and the sorted one give the same tokens the same result."""
    cfg = BM.config([att(window=1, mlp=moe(24, 5, (6, 3), 72, 40))], width=192, vocab=120, positions=320)
    w = BM.weights(cfg, 15)
    tok, want, _ = BM.clear_tokens(cfg, w, rows, 4)
    m = build(gpu, tmp_path, cfg, w, "bf16")
    a, b = feed(m, 1, tok, [rows]), feed(m, 2, tok, cut(rows, 7))
    assert err(a, want, "f32") < ONE["bf16"] and err(b, want, "f32") < ONE["bf16"]
    m.close()


@pytest.mark.parametrize("heads,kv_heads,dim,vdim,window", [(6, 2, 40, 24, None), (4, 1, 64, 128, 300), (20, 1, 20, 200, None)])
def test_key_splits(gpu, tmp_path, heads, kv_heads, dim, vdim, window):
    """Decoding and short portions with the keys split over workgroups: any number of splits, captured passes included."""
    cfg = BM.config([att(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, window=window), att(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, window=window, mlp=None)],
                    width=128, vocab=90, positions=460)
    w = BM.weights(cfg, 16)
    tok, want, _ = BM.clear_tokens(cfg, w, 450, 6)
    m = build(gpu, tmp_path, cfg, w, "bf16")
    lib = gpu.lib()
    try:
        for i, n in enumerate((1, 2, 3, 7, 16)):
            lib.nvl_set_tuning(37, n)
            assert err(feed(m, i, tok, [400] + [1] * 20 + [3] * 10), want, "bf16") < ONE["bf16"], n
            m.seq_close(i)
    finally:
        lib.nvl_set_tuning(37, 0)
    m.close()


def test_prompt_of_many_hundred_tokens(gpu, tmp_path):
    """Long enough that the narrow projections are split along K."""
    cfg = BM.config([att(window=40, mlp=None), att(window=40, mlp=moe(6, 2, None, 24))], width=520, vocab=90, side=30, positions=700)
    w = BM.weights(cfg, 18)
    tok, want, _ = BM.clear_tokens(cfg, w, 690, 6)
    m = build(gpu, tmp_path, cfg, w, "bf16")
    for i, cuts in enumerate(([690], [530, 160], [64, 600, 26])):
        assert err(feed(m, i, tok, cuts), want, "bf16") < ONE["bf16"], cuts
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
    """400 steps on the device for a batch of unequal sequences (captured passes) against the same steps one call at a time."""
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
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
def test_long_decoding(gpu, tmp_path, stack, precision):
    """300 tokens one by one behind a short prompt, in captured passes, beside a second sequence."""
    cfg, w, seqs, want = stack
    m = build(gpu, tmp_path, cfg, w, precision)
    m.seq_open(1)
    m.seq_open(2)
    m.forward_rows([1, 2], [seqs[0][:31], seqs[2][:3]], [0, 0], [])
    rows = [m.forward_batch([1, 2], [[seqs[0][31 + i]], [seqs[2][3 + i]]], [31 + i, 3 + i])[0] if i < 200 else m.forward_batch([1], [[seqs[0][31 + i]]], [31 + i])[0] for i in range(300)]
    assert err(np.stack([r[0] for r in rows]), want[0][31:], precision) < TOL[precision]
    assert err(np.stack([r[1] for r in rows[:200]]), want[2][3:], precision) < TOL[precision]
    assert m.stats()["graph_replays"] > 200
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
    """The sampler on this model's logits: top_k = 1 is the argmax, in the runner and in the fused loop; a draw follows the distribution."""
    cfg, w, seqs, want = stack
    m = build(gpu, tmp_path, cfg, w, "bf16")
    prompt = seqs[1][:50]
    greedy = m.greedy(prompt, 6, seq_id=1)
    m.seq_reset(2)
    lg, am = m.forward_batch([2], [prompt], [0])
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
    """examples/ask_greedy (the C consumer of the ABI) generates from a Bolinex folder."""
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
