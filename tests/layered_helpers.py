"""Shared by the tests of models described by a list of layers: building one on the device, feeding it in portions, and comparing its
logits with a plain restatement (`oracle`: the module with forward(cfg, weights, tokens))."""
from __future__ import annotations

import numpy as np

import potuzen_models as PM

TOL = {"f32": 1e-4, "bf16": 0.12}       # at any position: rms over the vocabulary of the difference / rms of the logits


def same_fields(L, got, want):
    """An nvl_layer_config of the library's reader against the fields the package's reader made."""
    for k, _ in got._fields_:
        g = getattr(got, k)
        if k == "decay":
            assert np.allclose(list(g), list(want[k]) + [0.0] * (L.MAX_DECAYS - len(want[k])), rtol=0, atol=1e-15), k
        else:
            assert (g == L.MIXER[want[k]]) if k == "mixer" else abs(g - want[k]) < 1e-6, (k, g, want[k])


def build(gpu, d, cfg, w, precision="f32", **kw):
    PM.write(d, cfg, w)
    kw = dict(dict(max_seq_len=1024, max_seqs=4, max_batch_tokens=1024, kv_num_blocks=64, kv_block_size=64, kv_pool=True), **kw)
    return gpu.HipTransformerModel.from_pretrained(str(d), precision=precision, **kw)


def err(got, want, precision="f32"):
    """The worst position.  bf16: leaving out 3 in 100 — a norm over a nearly vanishing vector (a Mamba-2 head whose C . B dt is close to
    -D, say) turns the rounding of its input into a flipped sign at single positions, in any implementation."""
    d = np.asarray(got, np.float64) - want
    e = np.sort((np.sqrt((d ** 2).mean(axis=-1)) / np.sqrt((want ** 2).mean())).reshape(-1))
    return float(e[-1 - (e.size * 3 // 100 if precision == "bf16" else 0)])


def steady(oracle, cfg, w, draw, limit=0.035):
    """Tokens from draw() on which the model is well conditioned: a norm over a nearly vanishing vector can blow up rounding at single
    positions, and tells nothing about the device.  Measured on the restatement, with the embeddings perturbed by a bf16 rounding."""
    e = np.asarray(w["embed"], np.float64)
    noisy = [dict(w, embed=e * (1 + np.random.default_rng(i).uniform(-1, 1, e.shape) * 2.0 ** -9)) for i in range(3)]
    for _ in range(100):
        tok = list(draw())
        want = oracle.forward(cfg, w, tok)
        if all(err(oracle.forward(cfg, n, tok), want) < limit for n in noisy):
            return tok, want
    raise AssertionError("no well-conditioned sequence found")


def feed(m, seq, tokens, cuts):
    """All logits of `tokens` fed in portions; the sequence stays open."""
    if m.seq_len(seq) < 0:
        m.seq_open(seq)
    out, at = [], m.seq_len(seq)
    for n in cuts:
        part = tokens[at:at + n]
        out.append(m.forward_rows([seq], [part], [at], range(len(part)))[0])
        at += n
    assert at == len(tokens)
    return np.concatenate(out)


def cut(total, n):
    return [n] * (total // n) + ([total % n] if total % n else [])


def greedy_oracle(oracle, cfg, w, prompt, n):
    tok, gaps = list(prompt), []
    for _ in range(n):
        last = oracle.forward(cfg, w, tok)[-1]
        lg = np.sort(last)
        gaps.append(lg[-1] - lg[-2])
        tok.append(int(last.argmax()))
    return tok[len(prompt):], min(gaps)


def mixed_run(m, seqs, want, plan, seed):
    """Runs the sequences numbered in `plan` through the model, up to four at a time: portions of some beside single tokens of others,
    sequences left out of steps, slots and blocks used again.  Returns (device logits, expected logits) of sampled rows."""
    g = np.random.default_rng(seed)
    live, todo, sid, seen, done = {}, list(plan), 100, [], 0
    while todo or live:
        while todo and len(live) < 4 and todo[0] not in {v[0] for v in live.values()}:
            live[sid] = [todo.pop(0), 0]
            m.seq_open(sid)
            sid += 1
        ids = [s for s in live if g.random() < 0.8] or list(live)[:1]
        toks, pos = [], []
        for s in ids:
            k, at = live[s]
            toks.append(seqs[k][at:at + int(g.choice([1, 1, 1, 2, 5, 16, 30, 64, 90]))])
            pos.append(at)
        total = sum(map(len, toks))
        rows = sorted(g.choice(total, min(total, 40), replace=False).tolist())
        got, am = m.forward_rows(ids, toks, pos, rows)
        assert np.array_equal(am, got.argmax(axis=1))
        seen.append((got, np.concatenate([want[live[s][0]][p:p + len(t)] for s, t, p in zip(ids, toks, pos)])[rows]))
        for s, t in zip(ids, toks):
            live[s][1] += len(t)
            if live[s][1] == len(seqs[live[s][0]]):
                live.pop(s)
                m.seq_close(s)
                done += 1
    assert done == len(plan)
    return np.concatenate([a for a, _ in seen]), np.concatenate([b for _, b in seen])
