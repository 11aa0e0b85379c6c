"""The Medulorn design on the device against its plain restatement (medulorn_oracle.py): each mechanism alone at sizes the kernels pad,
tile and split differently, prompts cut in every way, mixed batches, slots and blocks used again, keys far away, at block borders and at
the edges of chunks, windows and kept tokens, sinks of any size, long decoding, and generation through the framework's own entry points."""
import json
import os
import subprocess
import sys
from functools import partial
from pathlib import Path

import numpy as np
import pytest

import layered_helpers as H
import medulorn_models as MM
import medulorn_oracle as O
import potuzen_models as PM
from layered_helpers import TOL, build, cut, err, feed

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent
greedy_oracle = partial(H.greedy_oracle, O)
ONE = {"f32": 1e-4, "bf16": 0.03}       # a single layer
att, par, moe, rot = MM.attention, MM.parallel, MM.moe, MM.rot

SINGLE = {      # layer, width
    "odd": (att(), 96), "no-mask": (att(chunk=None), 96), "chunk-1": (att(chunk=1), 64), "chunk-63": (att(chunk=63), 64), "chunk-64": (att(chunk=64), 64), "chunk-65": (att(chunk=65), 64),
    "chunk-128": (att(chunk=128), 64), "chunk-long": (att(chunk=1000), 64), "no-turn": (att(turn=None), 64), "turn-2": (att(turn=rot(2, 50.0)), 64), "turn-all": (att(dim=32, vdim=32, turn=rot(32)), 64),
    "turn-18-of-26": (att(dim=26, turn=rot(18)), 64), "turn-scaled": (att(turn=rot(32, 800.0, (4.0, 1.0, 4.0, 64))), 64), "one-head-each": (att(heads=3, kv_heads=3), 96), "one-kv-head": (att(heads=5, kv_heads=1), 96),
    "group-34": (att(heads=34, kv_heads=1, dim=16, vdim=8, turn=rot(8)), 96), "group-70": (att(heads=70, kv_heads=1, dim=12, vdim=5, turn=rot(12), chunk=100), 64),
    "64-64": (att(heads=4, kv_heads=1, dim=64, vdim=64, chunk=None, turn=rot(64)), 128), "128-128": (att(heads=4, kv_heads=2, dim=128, vdim=128, turn=rot(64)), 128), "96-80": (att(heads=3, kv_heads=1, dim=96, vdim=80, turn=rot(96)), 128),
    "20-160": (att(heads=2, kv_heads=1, dim=20, vdim=160, turn=rot(20)), 64), "200-40": (att(heads=2, kv_heads=2, dim=200, vdim=40, turn=rot(100)), 64), "256-256": (att(heads=4, kv_heads=2, dim=250, vdim=256, scale=0.06), 96),
    "big-heads": (att(heads=2, kv_heads=1, dim=272, vdim=264, scale=0.05, turn=rot(136)), 64), "narrow": (att(heads=1, kv_heads=1, dim=4, vdim=4, turn=rot(4), mlp=MM.dense(5)), 12),
    "wide-row": (att(heads=2, kv_heads=1, mlp=MM.dense(16)), 1100), "negative-scale": (att(scale=-0.3), 64), "no-feed-forward": (att(mlp=None), 96), "dense-200": (att(mlp=MM.dense(200)), 70),
    "beside": (par(), 96), "beside-no-mask": (par(window=None), 96), "window-1": (par(window=1), 64), "window-1-keep-0": (par(window=1, keep=0), 64), "window-64": (par(window=64, keep=1), 64), "window-65-keep-64": (par(window=65, keep=64), 64),
    "keep-70": (par(window=20, keep=70), 64), "keep-more-than-all": (par(window=20, keep=400), 64), "beside-no-turn": (par(turn=None), 64), "beside-128": (par(heads=4, kv_heads=1, dim=128, vdim=128, heads2=2, dim2=128, vdim2=128, turn=rot(128)), 128),
    "beside-96-48": (par(heads=4, kv_heads=4, dim=48, vdim=96, heads2=5, dim2=32, vdim2=64, turn=rot(48)), 96), "lightning-odd": (par(heads2=1, dim2=7, vdim2=9), 64), "lightning-wide": (par(heads2=2, dim2=200, vdim2=150), 64),
    "lightning-huge": (par(heads2=1, dim2=300, vdim2=40), 64), "lightning-many": (par(heads2=40, dim2=8, vdim2=8), 64), "left-alone": (par(right_scale=0.0), 64), "right-alone": (par(left_scale=1e-6), 64), "beside-no-ff": (par(mlp=None), 64),
    "experts": (att(mlp=moe()), 96), "experts-no-shared": (att(mlp=moe(5, 2, 24, shared=None)), 64), "one-expert": (att(mlp=moe(1, 1, 24, shared=30)), 64), "experts-40": (att(mlp=moe(40, 6, 16, shared=8)), 64),
    "experts-72": (att(mlp=moe(72, 5, 12, shared=None)), 64), "experts-100-shared": (par(mlp=moe(100, 4, 12, shared=40)), 64), "every-expert": (att(mlp=moe(6, 6, 24)), 64), "wide-experts": (att(mlp=moe(6, 2, 200, shared=136)), 256),
    "shared-of-three": (att(mlp=moe(6, 2, 64, shared=180)), 64), "shared-of-many": (att(mlp=moe(6, 2, 16, shared=1100)), 64), "tight-limits": (att(mlp=moe(6, 2, 24, limit=0.3, shared=64, shared_limit=0.1)), 64),
}


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("name", list(SINGLE))
def test_one_layer(gpu, tmp_path, name, precision):
    """A mechanism alone: a prompt in one piece, then the same in portions of 20 with the last tokens one by one, and in pairs."""
    layer, width = SINGLE[name]
    cfg = MM.config([layer], width=width, vocab=130)
    w = MM.weights(cfg, 7)
    tok, want, layers = MM.clear_tokens(cfg, w, 149, 1)
    m = build(gpu, tmp_path, cfg, w, precision)
    m.set_debug(2)
    assert err(feed(m, 1, tok, [149]), want, precision) < ONE[precision]
    assert err(m.get_hidden(149), layers, precision) < ONE[precision]
    m.set_debug(0)
    assert err(feed(m, 2, tok, cut(129, 20) + [1] * 20), want, precision) < ONE[precision]
    assert err(feed(m, 3, tok, cut(149, 2)), want, precision) < ONE[precision]
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("over", [dict(alpha=1.0, scale=1.0, cap=None), dict(alpha=0.4, cap=3.0), dict(alpha=-1.3), dict(eps=0.3)])
def test_constants(gpu, tmp_path, over, precision):
    cfg = MM.config([att(), par(mlp=moe())], width=96, vocab=130, **over)
    w = MM.weights(cfg, 8)
    tok, want, _ = MM.clear_tokens(cfg, w, 120, 1)
    m = build(gpu, tmp_path, cfg, w, precision)
    for s, cuts in enumerate(([120], cut(100, 33) + [1] * 20)):
        assert err(feed(m, s, tok, cuts), want, precision) < 2 * ONE[precision]
    m.close()


def mixed_config():
    return MM.config([par(mlp=moe()), att(chunk=37), att(heads=4, kv_heads=2, dim=64, vdim=24, chunk=None, turn=rot(32), mlp=None), par(heads=2, kv_heads=1, dim=20, vdim=130, window=70, keep=66, turn=rot(20), heads2=2, dim2=64, vdim2=48, mlp=moe(8, 2, 72, shared=None)),
                      att(heads=12, kv_heads=2, dim=16, chunk=64, scale=0.5, turn=rot(16), mlp=moe(20, 4, 16, shared=100)), par(window=100, keep=0, mlp=None), att(heads=2, kv_heads=2, dim=100, chunk=96, turn=rot(96), mlp=MM.dense(200))],
                     width=168, vocab=259, eps=2e-6)


@pytest.fixture(scope="module")
def stack():
    """One model with every mechanism, and its logits for four sequences."""
    cfg = mixed_config()
    w = MM.weights(cfg, 21)
    both = [MM.clear_tokens(cfg, w, n, 5 + n) for n in (331, 70, 203, 6)]
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
@pytest.mark.parametrize("layers,blocks", [([att(chunk=70), att(chunk=20, mlp=moe(6, 2, 16, shared=8))], 4), ([par(window=70, keep=66), att(chunk=64)], 6), ([par(window=20, keep=0)], 3)])
def test_masks_give_blocks_back(gpu, tmp_path, layers, blocks, precision):
    """Chunks and windows in every layer: one long sequence runs in a pool of a few blocks, in portions and decoding, over blocks used
    again; blocks of kept tokens stay."""
    cfg = MM.config(layers, width=80, vocab=90)
    w = MM.weights(cfg, 9)
    tok, want, _ = MM.clear_tokens(cfg, w, 450, 2)
    m = build(gpu, tmp_path, cfg, w, precision, max_seqs=2, kv_num_blocks=blocks)
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


# ---- the token before: only the shift carries anything from one token to the next ----
@pytest.mark.parametrize("precision", ["f32", "bf16"])
def test_shift_alone(gpu, tmp_path, precision):
    """Chunks of one token: what a row knows of the tokens before it came through three layers of shift.  Cuts of every size, two sequences
    in turn and together, and a slot used again, whose kept rows must not be seen."""
    cfg = MM.config([att(chunk=1), att(chunk=1, mlp=None), att(chunk=1, mlp=moe(4, 2, 16, shared=8))], width=200, vocab=60)
    w = MM.weights(cfg, 11, shift=(0.6, 1.4))
    (a, want, _), (b, wantb, _) = MM.clear_tokens(cfg, w, 50, 1), MM.clear_tokens(cfg, w, 33, 2)
    swapped = list(a)
    swapped[20] = b[0]
    d = np.abs(O.forward(cfg, w, swapped) - want).max(axis=1)
    assert np.all(d[20:24] > 0.05) and np.all(d[24:] == 0) and np.all(d[:20] == 0)
    m = build(gpu, tmp_path, cfg, w, precision, max_seqs=2)
    for s, cuts in enumerate(([50], [1] * 50, cut(50, 2), cut(50, 3), [1, 2, 1, 4, 16, 1, 1, 17, 7], [33, 17])):
        assert err(feed(m, s, a, cuts), want, precision) < ONE[precision], cuts
        m.seq_close(s)
    m.seq_open(8)
    m.seq_open(9)
    got = {8: [], 9: []}
    at = {8: 0, 9: 0}
    for na, nb in ((3, 1), (1, 1), (1, 2), (16, 16), (2, 1), (1, 1), (1, 10), (25, 1)):
        lg, _ = m.forward_rows([9, 8], [b[at[9]:at[9] + nb], a[at[8]:at[8] + na]], [at[9], at[8]], range(na + nb))
        got[9].append(lg[:nb]); got[8].append(lg[nb:])
        at[8] += na; at[9] += nb
    assert err(np.concatenate(got[8]), want, precision) < ONE[precision] and err(np.concatenate(got[9]), wantb, precision) < ONE[precision]
    m.close()


# ---- single keys that stand out: far away, at block borders, at the edges of masks, the first tokens ----
def spotlight(cfg, w, A, B, score=24.0):
    """Queries of token B look for token A in every head of layer 0, wherever the two stand: their embeddings get a direction of their own,
    which W_q and W_k turn into one vector of the dimensions that do not turn; the norms make its length, the scale its score."""
    w = dict(w)
    ly, W = cfg["layers"][0], cfg["width"]
    two = ly["type"] == "parallel"
    mx, p = (ly["mixer"]["left"], "l0.mix.left.") if two else (ly["mixer"], "l0.mix.")
    turn = (mx.get("rot") or dict(dims=0))["dims"]
    assert abs(mx["scale"] * mx["dim"] / score - 1) < 1e-6 and turn + 8 <= mx["dim"]
    g = np.random.default_rng(99)
    u, v = np.linalg.qr(g.standard_normal((W, 2)))[0].T
    w["embed"] = PM.bf16(w["embed"] - (w["embed"] @ np.stack([u, v]).T) @ np.stack([u, v]))      # (a direction nobody else has: the norms hide how little it is)
    w["embed"][A], w["embed"][B] = PM.bf16(3 * u), PM.bf16(3 * v)
    w["l0.shift"] = np.zeros_like(w["l0.shift"])
    h = {t: w["embed"][t].astype(np.float64) * cfg["embedding"]["scale"] for t in (A, B)}
    k = np.concatenate([np.zeros((mx["kv_heads"], turn)), g.choice([-1.0, 1.0], (mx["kv_heads"], mx["dim"] - turn))], axis=1)
    q = np.repeat(k, mx["heads"] // mx["kv_heads"], axis=0)
    for n, x, t in (("k", k, A), ("q", q, B)):
        w[p + n] = PM.bf16(w[p + n] + 60.0 * np.outer(x.reshape(-1), h[t] / (h[t] @ h[t])))
        w[p + n + ".norm"] = np.ones_like(w[p + n + ".norm"])
        if p + n + ".b" in w:
            w[p + n + ".b"] = PM.bf16(0.1 * w[p + n + ".b"])
    w[p + "o"] = PM.bf16(12.0 * w[p + "o"])                                  # (what attention brings should show beside the stream)
    return w


def spot_layer(kind, **kw):
    if kind == "chunk":
        return att(**dict(dict(heads=4, kv_heads=2, dim=32, vdim=32, turn=rot(16), scale=24.0 / 32, mlp=None), **kw))
    return par(**dict(dict(heads=4, kv_heads=2, dim=32, vdim=32, turn=rot(16, 500.0, (4.0, 1.0, 4.0, 100)), scale=24.0 / 32, right_scale=0.0, mlp=None), **kw))


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("kind,kw", [("chunk", dict(chunk=None, heads=17, kv_heads=1)), ("chunk", dict(chunk=700, dim=72, vdim=40, scale=24.0 / 72)), ("window", dict(window=700, keep=4))])
def test_far_key_among_hundreds(gpu, tmp_path, kind, kw, precision):
    A, B, V = 77, 88, 90
    cfg = MM.config([spot_layer(kind, **kw)], width=128, vocab=V)
    w = spotlight(cfg, MM.weights(cfg, 43), A, B)
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
            assert err(got[[600, 639]], want[[600, 639]], precision) < 2 * ONE[precision], (at, cuts)
            m.seq_close(10 * i + len(cuts))
    m.close()


def edge_case(gpu, m, cfg, w, A, B, V, n, q, inside, outside, sid, precision):
    """Token B at q, token A at `inside` or `outside`: what is outside leaves no trace in row q, what is inside decides it."""
    g = np.random.default_rng(9 + q)
    base = g.integers(0, A, n)
    base[q] = B
    rows = {}
    for name, at in (("in", inside), ("out", outside)):
        if at is None:
            continue
        tok = base.copy()
        tok[at] = A
        tok = tok.tolist()
        want = O.forward(cfg, w, tok)
        for cuts in ([n], [q] + [1] * (n - q), [q - 20, 21, n - 1 - q] if q < n - 1 else cut(n, 2)):
            got = feed(m, sid[0], tok, cuts)
            assert err(got[[q]], want[[q]], precision) < 3 * ONE[precision], (q, name, cuts)
            m.seq_close(sid[0])
            sid[0] += 1
        rows[name] = want[q]
    plain = O.forward(cfg, w, base.tolist())[q]
    if "out" in rows:
        assert np.allclose(rows["out"], plain, atol=1e-12)
    if "in" in rows:
        assert err(rows["in"][None], plain[None]) > 0.3


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("chunk", [2, 31, 64, 65, 100, 192])
def test_chunk_edges(gpu, tmp_path, chunk, precision):
    """The first key of a query's chunk and the last of the chunk before, for queries at both ends of chunks and between."""
    A, B, V, n = 77, 88, 90, 320
    cfg = MM.config([spot_layer("chunk", chunk=chunk)], width=96, vocab=V)
    w = spotlight(cfg, MM.weights(cfg, 44), A, B)
    m = build(gpu, tmp_path, cfg, w, precision)
    sid = [0]
    c0 = 200 // chunk * chunk
    for q in {c0, min(c0 + 1, n - 1), c0 - 1, 255, 256, 301, 319}:
        first = q // chunk * chunk
        edge_case(gpu, m, cfg, w, A, B, V, n, q, first if first < q else None, first - 1 if first > 0 else None, sid, precision)
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("window,keep", [(1, 0), (2, 1), (31, 5), (64, 64), (65, 3), (100, 70), (192, 0)])
def test_window_and_kept_edges(gpu, tmp_path, window, keep, precision):
    """The last key inside a window and the first outside; the last of the kept tokens and the first behind them."""
    A, B, V, n = 77, 88, 90, 320
    cfg = MM.config([spot_layer("window", window=window, keep=keep)], width=96, vocab=V)
    w = spotlight(cfg, MM.weights(cfg, 45), A, B)
    m = build(gpu, tmp_path, cfg, w, precision)
    sid = [0]
    for q in (200, 255, 256, 301, 319):
        back = q - window
        edge_case(gpu, m, cfg, w, A, B, V, n, q, back + 1 if window > 1 else None, back if back >= keep else None, sid, precision)
        if 0 < keep <= back:
            edge_case(gpu, m, cfg, w, A, B, V, n, q, keep - 1, keep if keep < back else None, sid, precision)
    if keep:
        edge_case(gpu, m, cfg, w, A, B, V, n, 300, 0, None, sid, precision)
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("sink", [(-60.0, 1.0), (0.0, 3.0), (9.0, 2.0), (300.0, 1.0)])
def test_sinks_of_any_size(gpu, tmp_path, sink, precision):
    """Sinks that nothing reaches, that compete, and that take everything; the restatement without them, or with them scaled, is elsewhere."""
    cfg = MM.config([par(window=40, keep=2, right_scale=0.0, scale=0.9, mlp=None)], width=96, vocab=70)
    w = MM.weights(cfg, 48, sink=sink)
    w["l0.mix.left.o"] = PM.bf16(4 * w["l0.mix.left.o"])
    tok = np.random.default_rng(10).integers(0, 70, 200).tolist()
    want = O.forward(cfg, w, tok)
    if sink[0] == 9.0:
        assert err(O.forward(cfg, dict(w, **{"l0.mix.left.sink": w["l0.mix.left.sink"] * 0.9}), tok), want) > 0.02
    m = build(gpu, tmp_path, cfg, w, precision)
    for s, cuts in enumerate(([200], [150] + [1] * 50, cut(200, 33))):
        assert err(feed(m, s, tok, cuts), want, precision) < ONE[precision]
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
def test_a_one_in_the_denominator(gpu, tmp_path, precision):
    """Strongly negative scores: the one outweighs the keys, and a softmax without it would be far away."""
    cfg = MM.config([att(chunk=40, heads=2, kv_heads=1, dim=16, vdim=32, turn=None, scale=-0.6, mlp=None)], width=64, vocab=70)
    w = MM.weights(cfg, 49)
    w["l0.mix.k"], w["l0.mix.q"] = PM.bf16(0.1 * w["l0.mix.k"]), PM.bf16(0.1 * w["l0.mix.q"])
    b = np.random.default_rng(1).choice([-1.0, 1.0], 16)
    w["l0.mix.k.b"], w["l0.mix.q.b"] = PM.bf16(b), PM.bf16(np.tile(b, 2))
    w["l0.mix.o"] = PM.bf16(8 * w["l0.mix.o"])
    tok = np.random.default_rng(10).integers(0, 70, 130).tolist()
    want = O.forward(cfg, w, tok)
    keep = O.sink_softmax
    try:
        O.sink_softmax = lambda s, sink: keep(s, sink - 1e9)
        assert err(O.forward(cfg, w, tok), want) > 0.3
    finally:
        O.sink_softmax = keep
    m = build(gpu, tmp_path, cfg, w, precision)
    for s, cuts in enumerate(([130], [100] + [1] * 30, cut(130, 3))):
        assert err(feed(m, s, tok, cuts), want, precision) < ONE[precision]
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
def test_rotation_far_along(gpu, tmp_path, precision):
    """Thousands of positions: angles of every pair, with and without stretched waves; the restatement one position off is far away."""
    cfg = MM.config([att(heads=2, kv_heads=1, dim=32, vdim=32, chunk=None, turn=rot(32, 3e4), scale=0.6, mlp=None), par(heads=2, kv_heads=1, dim=32, vdim=32, window=1500, turn=rot(32, 3e4, (6.0, 1.0, 4.0, 700)), scale=0.6, mlp=None)], width=64, vocab=70)
    w = MM.weights(cfg, 50)
    tok = np.random.default_rng(3).integers(0, 70, 2100).tolist()
    want = O.forward(cfg, w, tok)
    m = build(gpu, tmp_path, cfg, w, precision, max_seq_len=2200, max_batch_tokens=2200)
    got = feed(m, 1, tok, [1300, 780] + [1] * 20)
    assert err(got, want, precision) < 2 * ONE[precision]
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("decay", [[0.0, 1.0, 0.9999], [0.3, 0.02, 0.999], [1e-6, 0.5, 1.0]])
def test_lightning_decays(gpu, tmp_path, decay, precision):
    """Decays from nothing to one, over a prompt in parallel pieces, short portions and single tokens."""
    cfg = MM.config([par(left_scale=1e-6, heads2=3, dim2=20, vdim2=28, decay=decay, right_scale=2.0, mlp=None)], width=96, vocab=70)
    w = MM.weights(cfg, 51)
    tok = np.random.default_rng(4).integers(0, 70, 900).tolist()
    want = O.forward(cfg, w, tok)
    m = build(gpu, tmp_path, cfg, w, precision)
    for s, cuts in enumerate(([900], [560, 5, 4, 3, 2, 1, 301] + [1] * 24, cut(900, 97))):
        assert err(feed(m, s, tok, cuts), want, precision) < ONE[precision], cuts
        m.seq_close(s)
    m.close()


@pytest.mark.parametrize("rows", [64, 65, 100, 300])
@pytest.mark.parametrize("shared", [40, 200, 1300])
def test_expert_forms_agree(gpu, tmp_path, rows, shared):
    """The masked form (up to 64 rows a call, the shared expert among the others or by itself) and the sorted one give the same result."""
    cfg = MM.config([att(chunk=1, mlp=moe(24, 5, 72, shared=shared))], width=192, vocab=120)
    w = MM.weights(cfg, 15)
    tok, want, _ = MM.clear_tokens(cfg, w, rows, 4)
    m = build(gpu, tmp_path, cfg, w, "bf16")
    a, b = feed(m, 1, tok, [rows]), feed(m, 2, tok, cut(rows, 7))
    assert err(a, want, "f32") < ONE["bf16"] and err(b, want, "f32") < ONE["bf16"]
    m.close()


@pytest.mark.parametrize("layer", [att(chunk=None), att(heads=4, kv_heads=1, dim=64, vdim=128, chunk=300), par(heads=20, kv_heads=1, dim=20, vdim=200, window=None, turn=rot(20)), par(window=200, keep=70)])
def test_key_splits(gpu, tmp_path, layer):
    """Decoding and short portions with the keys split over workgroups: any number of splits, captured passes included."""
    cfg = MM.config([layer, dict(layer, mlp=None)], width=128, vocab=90)
    w = MM.weights(cfg, 16)
    tok, want, _ = MM.clear_tokens(cfg, w, 450, 6)
    m = build(gpu, tmp_path, cfg, w, "bf16")
    lib = gpu.lib()
    try:
        for i, n in enumerate((1, 2, 3, 7, 16)):
            lib.nvl_set_tuning(37, n)
            assert err(feed(m, i, tok, [400] + [1] * 20 + [3] * 10), want, "bf16") < 1.5 * ONE["bf16"], n
            m.seq_close(i)
    finally:
        lib.nvl_set_tuning(37, 0)
    m.close()


def test_prompt_of_many_hundred_tokens(gpu, tmp_path):
    """Long enough for the kernels of whole row tiles: norms of sums, shift, query/key norms and rotation, experts gathered."""
    cfg = MM.config([att(chunk=40), par(window=40, mlp=moe(6, 2, 24))], width=520, vocab=90)
    w = MM.weights(cfg, 18)
    tok, want, _ = MM.clear_tokens(cfg, w, 690, 6)
    m = build(gpu, tmp_path, cfg, w, "bf16")
    for i, cuts in enumerate(([690], [530, 160], [64, 600, 26])):
        assert err(feed(m, i, tok, cuts), want, "bf16") < 1.5 * ONE["bf16"], cuts
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
    """400 steps on the device for a batch of unequal sequences (captured passes) against the same steps one call at a time; then both go on
    with a portion, whose first token needs the row the loop left behind."""
    cfg, w, seqs, _ = stack
    m = build(gpu, tmp_path, cfg, w, "bf16", max_seqs=3, kv_num_blocks=30)
    prompts, first = [seqs[0][:90], seqs[1][:7], seqs[2][:64]], []
    for i, p in enumerate(prompts):
        m.seq_open(i)
        first.append(int(m.forward_batch([i], [p], [0])[1][0]))
    out = m.decode_greedy([0, 1, 2], first, 400)
    more = [[int(out[-1, i]), 5, 6] for i in range(3)]
    behind = m.forward_rows([0, 1, 2], more, [len(p) + 400 for p in prompts], range(9))[0]
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
    assert np.array_equal(m.forward_rows([10, 11, 12], more, [len(p) + 400 for p in prompts], range(9))[0], behind)
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
    """examples/ask_greedy (the C consumer of the ABI) generates from a Medulorn folder."""
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
