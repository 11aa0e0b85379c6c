"""The Potuzen design on the device against its plain restatement (potuzen_oracle.py): each mechanism alone at sizes the kernels pad,
tile and split differently, prompts cut in every way, mixed batches, slots and blocks used again, keys at window and block
borders, long decoding, and generation through the framework's own entry points."""
import json
import os
import subprocess
import sys
from functools import partial
from pathlib import Path

import numpy as np
import pytest

import layered_helpers as H
import potuzen_models as PM
import potuzen_oracle as O
from layered_helpers import TOL, build, cut, err, feed

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent
steady, greedy_oracle = partial(H.steady, O), partial(H.greedy_oracle, O)

SINGLE = {
    "latent-odd": (PM.latent(), 96), "latent-64": (PM.latent(heads=6, dim=64, vdim=64, q_rank=96, kv_rank=64, window=64), 128),
    "latent-window-1": (PM.latent(window=1), 64), "latent-window-2": (PM.latent(window=2, dim=32, vdim=32), 64),
    "latent-wide-window": (PM.latent(heads=2, dim=100, vdim=130, kv_rank=128, window=900), 64),
    "latent-17-heads": (PM.latent(heads=17, dim=16, vdim=8, kv_rank=256, window=33, scale=1.0), 96),
    "latent-kv-320": (PM.latent(heads=1, dim=8, vdim=16, q_rank=5, kv_rank=320, window=130), 200),
    "latent-kv-512": (PM.latent(heads=4, dim=128, vdim=128, q_rank=192, kv_rank=512, window=100), 256),
    "latent-not-absorbable": (PM.latent(heads=2, dim=64, vdim=64, kv_rank=576, window=70), 64),
    "latent-big-heads": (PM.latent(heads=2, dim=272, vdim=264, window=77, scale=0.06), 64),
    "latent-negative-scale": (PM.latent(scale=-0.4, window=40), 64),
    "mamba-odd": (PM.mamba2(), 96), "mamba-64": (PM.mamba2(heads=4, vdim=64, state=128, groups=1, norm_groups=4, conv=4), 128),
    "mamba-conv-1": (PM.mamba2(heads=3, vdim=33, state=16, groups=3, norm_groups=3, conv=1), 64),
    "mamba-conv-7": (PM.mamba2(heads=6, vdim=18, state=40, groups=2, norm_groups=2, conv=7), 70),
    "mamba-wide-heads": (PM.mamba2(heads=2, vdim=200, state=64, groups=1, norm_groups=1, conv=2), 64),
    "mamba-state-300": (PM.mamba2(heads=2, vdim=16, state=300, groups=1, conv=4), 64),
    "mamba-long-norm": (PM.mamba2(heads=8, vdim=80, state=16, groups=4, norm_groups=1, conv=4), 64),
    "gla-odd": (PM.gla(), 96), "gla-128": (PM.gla(heads=2, dim=128, vdim=128, tau=16.0), 128),
    "gla-wide-values": (PM.gla(heads=2, dim=64, vdim=200, tau=4.0), 64), "gla-200": (PM.gla(heads=1, dim=200, vdim=70, tau=8.0), 64),
    "gla-300": (PM.gla(heads=1, dim=300, vdim=20), 64), "gla-tau": (PM.gla(heads=3, dim=10, vdim=6, tau=0.3), 36),
    "no-feed-forward": (PM.gla(ff=None), 96), "wide-row": (PM.gla(heads=1, dim=16, vdim=16, ff=16), 1100),
    "narrow": (PM.latent(heads=1, dim=4, vdim=4, q_rank=3, kv_rank=2, ff=5, window=9), 12),
}


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("name", list(SINGLE))
def test_one_layer(gpu, tmp_path, name, precision):
    """A mechanism alone: a prompt in one piece, then the same in portions of 20 with the last tokens one by one."""
    layer, width = SINGLE[name]
    cfg = PM.config([layer], width=width, vocab=130)
    w = PM.weights(cfg, 7, rank=8 if name != "gla-200" else 40)
    g = np.random.default_rng(1)
    tok, want = steady(cfg, w, lambda: g.integers(0, 130, 149).tolist())
    layers = O.forward(cfg, w, tok, return_layers=True)[1]
    m = build(gpu, tmp_path, cfg, w, precision)
    m.set_debug(2)
    assert err(feed(m, 1, tok, [149]), want, precision) < TOL[precision]
    assert err(m.get_hidden(149), layers, precision) < TOL[precision]
    m.set_debug(0)
    assert err(feed(m, 2, tok, cut(129, 20) + [1] * 20), want, precision) < TOL[precision]
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("decay_bias,tau", [(-30.0, 0.5), (30.0, 16.0), (-4.0, 16.0)])
def test_gla_decay_extremes(gpu, tmp_path, decay_bias, tau, precision):
    """Decays close to 0 (a factor e^-60 per token and below: exponentials of the opposite sign would overflow inside a chunk) and
    close to 1 (nothing is forgotten)."""
    cfg = PM.config([PM.gla(heads=4, dim=48, vdim=40, tau=tau)], width=96, vocab=90)
    w = PM.weights(cfg, 11, decay_bias=decay_bias)
    tok = np.random.default_rng(2).integers(0, 90, 200).tolist()
    want = O.forward(cfg, w, tok)
    m = build(gpu, tmp_path, cfg, w, precision)
    for cuts in ([200], cut(200, 37), [180] + [1] * 20):
        got = feed(m, len(cuts), tok, cuts)
        # (with everything forgotten a head's output is (q . k) v, whose norm flips its sign where q . k vanishes: the median position)
        e = np.sqrt(((got - want) ** 2).mean(axis=1)) / np.sqrt((want ** 2).mean())
        assert np.isfinite(got).all() and np.median(e) < (5e-6 if precision == "f32" else 0.03) and np.sort(e)[-10] < TOL[precision]
    m.close()


def mixed_config():
    return PM.config([PM.latent(window=50), PM.mamba2(), PM.gla(), PM.latent(heads=2, dim=64, vdim=48, kv_rank=40, window=130, ff=None),
                      PM.mamba2(heads=2, vdim=64, state=32, groups=1, norm_groups=2, conv=4, ff=200), PM.latent(window=50, weights_of=0),
                      PM.gla(weights_of=2)], width=168, vocab=259, eps=2e-6)


@pytest.fixture(scope="module")
def stack():
    """One model with every mechanism, two windows and shared tensors, and its logits for four sequences."""
    cfg = mixed_config()
    w = PM.weights(cfg, 21)
    g = np.random.default_rng(5)
    both = [steady(cfg, w, lambda n=n: g.integers(0, 259, n).tolist()) for n in (331, 70, 203, 6)]
    return cfg, w, [b[0] for b in both], [b[1] for b in both]


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("cuts", ["whole", "ones", "twos", "3", "16", "17", "63", "64", "65", "128", "ragged", "tail"])
def test_portions(gpu, tmp_path, stack, cuts, precision):
    cfg, w, seqs, want = stack
    n = len(seqs[0])
    plan = dict(whole=[n], ones=[1] * n, twos=cut(n, 2), ragged=[2, 64, 3, 1, 1, 29, 128, 5, 16, 50, 32], tail=[n - 60] + [1] * 60).get(cuts) or cut(n, int(cuts))
    m = build(gpu, tmp_path, cfg, w, precision)
    assert err(feed(m, 3, seqs[0], plan), want[0], precision) < TOL[precision]
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
def test_long_prompts_in_parallel_pieces(gpu, tmp_path, precision):
    """Few heads and a long portion: the recurrences run piece by piece in parallel (three launches), from a zero and from a carried state."""
    cfg = PM.config([PM.gla(heads=2, dim=40, vdim=72), PM.mamba2(heads=4, vdim=32, state=24, groups=2, conv=4), PM.latent(window=300)], width=96, vocab=100)
    w = PM.weights(cfg, 31, decay_bias=3.0)
    tok = np.random.default_rng(3).integers(0, 100, 1500).tolist()
    want = O.forward(cfg, w, tok)
    m = build(gpu, tmp_path, cfg, w, precision, max_seq_len=1536, max_batch_tokens=1536)
    for cuts in ([1500], [600, 5, 700, 195], [513] + [1] * 7 + [980]):
        assert err(feed(m, len(cuts), tok, cuts), want, precision) < TOL[precision]
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
def test_mixed_batches_and_reuse(gpu, tmp_path, stack, precision):
    """Portions of some sequences beside single tokens of others, sequences left out of steps, slots and blocks given back and used
    again: every logit as if the sequence were alone.  The pool is exactly as large as the live sequences need."""
    cfg, w, seqs, want = stack
    need = sum(-(-len(s) // 64) for s in seqs)
    m = build(gpu, tmp_path, cfg, w, precision, max_seqs=4, kv_num_blocks=need)
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


# ---- single keys that stand out: windows, borders, first tokens ----
def spotlight(cfg, w, A, B, score=30.0):
    """Queries of token B look for token A: W_uq gets a term that adds `score` to that one score in every head."""
    w = dict(w)
    mx, eps = cfg["layers"][0]["mixer"], cfg["norm"]["eps"]
    H, d = mx["heads"], mx["dim"]
    h = {t: O.rms_norm(np.asarray(w["embed"][t], np.float64), w["l0.norm1"], eps) for t in (A, B)}
    cq = O.rms_norm(w["l0.mix.dq"] @ h[B], w["l0.mix.dq.norm"], eps)
    k = (w["l0.mix.uk"] @ O.rms_norm(w["l0.mix.dkv"] @ h[A], w["l0.mix.dkv.norm"], eps)).reshape(H, d)
    uq = np.array(w["l0.mix.uq"], np.float64).reshape(H, d, -1)
    for i in range(H):
        uq[i] += np.outer(k[i] * (score / mx["scale"] / (k[i] @ k[i])), cq / (cq @ cq))
    w["l0.mix.uq"] = PM.bf16(uq.reshape(H * d, -1))
    return w


@pytest.mark.parametrize("precision", ["f32", "bf16"])
@pytest.mark.parametrize("window", [31, 64, 65, 136])
def test_window_edges(gpu, tmp_path, window, precision):
    """A key just inside and just outside the window of a query that looks for it, at block borders and at position 0, in a prompt, in
    portions that end between the two, and decoded.  The restatement with a window one token off must be far away."""
    A, B, V = 77, 88, 90
    cfg = PM.config([PM.latent(heads=2, dim=32, vdim=40, q_rank=64, kv_rank=64, window=window, scale=0.2, ff=None)], width=128, vocab=V)
    w = spotlight(cfg, PM.weights(cfg, 41), A, B)
    off = {s: dict(cfg, layers=[PM.latent(heads=2, dim=32, vdim=40, q_rank=64, kv_rank=64, window=window + s, scale=0.2, ff=None)]) for s in (1, -1)}
    m = build(gpu, tmp_path, cfg, w, precision)
    g, sid = np.random.default_rng(6), 0
    for at in (0, 1, 63, 64, 100):
        for inside in (True, False):
            q = at + window - 1 + (not inside)
            tok = g.integers(0, A, q + 1)
            tok[at], tok[q] = A, B
            tok = tok.tolist()
            want = O.forward(cfg, w, tok)
            wrong = O.forward(off[-1 if inside else 1], w, tok)
            assert err(wrong[q:], want[q:]) > 0.5
            for cuts in ([q + 1], [q, 1], cut(q + 1, 50), [max(q - 3, 1), q + 1 - max(q - 3, 1)]):
                assert err(feed(m, sid, tok, [c for c in cuts if c])[q:], want[q:], precision) < TOL[precision], (at, inside, cuts)
                m.seq_close(sid)
                sid += 1
    m.close()


@pytest.mark.parametrize("precision", ["f32", "bf16"])
def test_far_key_among_hundreds(gpu, tmp_path, precision):
    A, B, V = 77, 88, 90
    cfg = PM.config([PM.latent(heads=17, dim=16, vdim=16, q_rank=48, kv_rank=128, window=700, scale=0.5, ff=None)], width=128, vocab=V)
    w = spotlight(cfg, PM.weights(cfg, 43), A, B)
    m = build(gpu, tmp_path, cfg, w, precision)
    g = np.random.default_rng(8)
    for i, at in enumerate((0, 5, 127, 128, 300)):
        tok = g.integers(0, A, 640)
        tok[at], tok[600], tok[639] = A, B, B
        tok = tok.tolist()
        want = O.forward(cfg, w, tok)
        gone = list(tok)
        gone[at] = 3
        assert err(O.forward(cfg, w, gone)[639:], want[639:]) > 0.5
        got = feed(m, i, tok, [590, 40] + [1] * 10)
        assert err(got[[600, 639]], want[[600, 639]], precision) < TOL[precision]
        m.seq_close(i)
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
    """400 steps on the device for a batch of unequal sequences (captured passes, blocks taken ahead and given back as windows move on)
    against the same steps one call at a time; the last logits against the restatement of what was generated."""
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


def test_pool_limits(gpu, tmp_path):
    """An empty pool is an error that leaves the open sequences usable; with windows on every attention layer a sequence far longer than
    the pool runs through it."""
    cfg = PM.config([PM.latent(window=100), PM.mamba2()], width=64, vocab=80)
    w = PM.weights(cfg, 51)
    m = build(gpu, tmp_path, cfg, w, kv_num_blocks=4, max_seqs=2)
    tok = np.random.default_rng(9).integers(0, 80, 900).tolist()
    want = O.forward(cfg, w, tok)
    m.seq_open(1)
    m.seq_open(2)
    m.forward_rows([2], [tok[:64]], [0], [])
    with pytest.raises(gpu.NvlError) as e:
        m.forward_rows([1], [tok[:256]], [0], [0])
    assert e.value.code == -4
    assert err(m.forward_rows([2], [tok[64:70]], [64], range(6))[0], want[64:70]) < TOL["f32"]
    m.seq_close(2)
    assert err(feed(m, 1, tok, cut(900, 60)), want) < TOL["f32"]
    m.close()


def test_pool_serves_the_other_families(gpu):
    """kv_pool: the library's block allocator under the slot calls, same logits as one slab per slot — also for a hybrid with slot state."""
    for family in ("llama", "granite_hybrid"):
        cfg = gpu.synth.tiny_config(family)
        w = gpu.synth.make_weights(cfg, seed=5, scale=0.05)
        g = np.random.default_rng(4)
        prompts = [g.integers(0, cfg["vocab_size"], n).tolist() for n in (100, 33)]
        out = []
        for kw in (dict(), dict(kv_num_blocks=4, kv_block_size=64, kv_pool=True)):
            m = gpu.HipTransformerModel(cfg, w, precision="f32", max_seqs=2, max_batch_tokens=256, **kw)
            for s in (1, 2):
                m.seq_reset(s)
            lg, am = m.forward_batch([1, 2], prompts, [0, 0])
            toks = m.decode_greedy([1, 2], am, 6)
            m.seq_close(1)
            m.seq_open(3)
            l2, _ = m.forward_batch([3], [prompts[0]], [0])
            out.append((lg, toks, l2))
            m.close()
        for a, b in zip(*out):
            assert np.array_equal(a, b), family


def test_command_line(gpu, tmp_path, stack):
    """examples/ask_greedy (the C consumer of the ABI) generates from a Potuzen folder."""
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
