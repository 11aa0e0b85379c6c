"""The Potuzen design on the CPU: both readers of its config.json, what they refuse, and the plain restatement (potuzen_oracle.py)
against properties it must have."""
import ctypes as C
import json

import numpy as np
import pytest

import potuzen_models as PM
import potuzen_oracle as O
from layered_helpers import same_fields


def three_kinds():
    return PM.config([PM.latent(), PM.mamba2(), PM.gla(), PM.latent(weights_of=0), PM.gla(ff=None)], width=144, vocab=211, eps=3e-6)


def test_readers_agree(pkg, tmp_path):
    L, raw = pkg._lib, three_kinds()
    p = tmp_path / "config.json"
    p.write_text(json.dumps(raw))
    c = L.ModelConfigC()
    L.check(L.lib().nvl_load_config_json(str(p).encode(), C.byref(c)))
    want = pkg.config.load_model_config(raw)
    assert (c.vocab_size, c.hidden, c.num_layers, c.max_seq_len) == (211, 144, 5, 4096) == (want.vocab_size, want.hidden, want.num_layers, want.max_seq_len)
    assert abs(c.norm_eps - 3e-6) < 1e-12 and want.norm_eps == 3e-6
    assert c.activation_type == L.ACT[want.activation_type] == 2 and c.block_style == L.BLOCK[want.block_style] == 2
    n = L.lib().nvl_load_layers_json(str(p).encode(), None, 0)
    arr = (L.LayerConfigC * n)()
    assert L.lib().nvl_load_layers_json(str(p).encode(), arr, n) == n == len(want.layers)
    for a, w in zip(arr, want.layers):
        same_fields(L, a, w)
    assert arr[3].weights_of == 0 and arr[0].weights_of == -1 and arr[4].ffn_dim == 0 and arr[0].window == 50


def test_readers_refuse_what_they_do_not_know(pkg, tmp_path):
    L = pkg._lib
    p = tmp_path / "config.json"
    for change in (dict(layers=[]), dict(width=None), dict(layers=[dict(type="rwkv", mixer=dict(heads=1, vdim=1), mlp=None)]),
                   dict(layers=[dict(PM.gla(), mlp=dict(kind="sparse", ff=8))]), dict(norm={})):
        p.write_text(json.dumps(dict(three_kinds(), **change)))
        c = L.ModelConfigC()
        assert L.lib().nvl_load_config_json(str(p).encode(), C.byref(c)) == -1, change
    p.write_text(json.dumps(dict(model_type="llama", hidden_size=512)))
    assert L.lib().nvl_load_layers_json(str(p).encode(), None, 0) == 0          # every other architecture: no list


def test_create_refuses_bad_lists_before_touching_a_device(pkg):
    L = pkg._lib
    from importlib import import_module
    M = import_module("nano-vllm-go_amd.model")
    opts = L.RuntimeOptsC(device=0, precision=0, max_seqs=2, tp_size=1)
    h = C.c_void_p()
    good = [PM.latent(), PM.gla()]
    for layers in ([PM.latent(weights_of=1), PM.gla()], [PM.gla(weights_of=1), PM.gla(weights_of=0)], [PM.mamba2(heads=4, groups=3)],
                   [PM.mamba2(norm_groups=7)], [PM.gla(), PM.gla(dim=20, weights_of=0)], [PM.gla(tau=0.0)]):
        cfg = pkg.config.load_model_config(PM.config(layers)).to_dict()
        rc = L.lib().nvl_create_layers(C.byref(M._cfg_struct(cfg)), M._layer_structs(cfg["layers"]), C.byref(opts), C.byref(h))
        assert rc == -1, layers
    cfg = pkg.config.load_model_config(PM.config(good)).to_dict()
    c = M._cfg_struct(cfg)
    assert L.lib().nvl_create(C.byref(c), C.byref(opts), C.byref(h)) == -1          # needs its layer list
    bad = L.RuntimeOptsC(device=0, precision=0, max_seqs=0, tp_size=1)
    assert L.lib().nvl_create_layers(C.byref(c), M._layer_structs(cfg["layers"]), C.byref(bad), C.byref(h)) == -1


# ---- the plain restatement ----
def test_oracle_window_and_causality():
    cfg = PM.config([PM.latent(window=7, ff=None)], width=96, vocab=50)
    w = PM.weights(cfg, 3)
    t = np.random.default_rng(0).integers(0, 50, 30)
    a = O.forward(cfg, w, t)
    b = t.copy()
    b[10] = (b[10] + 1) % 50
    d = np.abs(O.forward(cfg, w, b) - a).max(axis=1)
    assert np.all(d[:10] == 0) and np.all(d[10:17] > 1e-6) and np.all(d[17:] == 0)       # seen by itself and the 6 after it


def test_oracle_recurrences_against_closed_forms():
    g = np.random.default_rng(1)
    T, H, d, dv = 9, 2, 5, 3
    q, k, v = g.standard_normal((T, H, d)), g.standard_normal((T, H, d)), g.standard_normal((T, H, dv))
    la = -g.uniform(0, 2, (T, H, d))
    b = np.cumsum(la, axis=0)
    want = np.zeros((T, H, dv))
    for t in range(T):
        for s in range(t + 1):
            want[t] += np.einsum("hd,hd,hd->h", q[t], k[s], np.exp(b[t] - b[s]))[:, None] * v[s]
    assert np.allclose(O.gla_recurrence(q, k, v, la), want)
    dt, A, D = g.uniform(0.1, 1, (T, H)), g.standard_normal(H), g.standard_normal(H)
    B, Cc = g.standard_normal((T, 1, d)), g.standard_normal((T, 1, d))
    got = O.ssd_recurrence(v, B, Cc, dt, A, D)
    s = np.cumsum(-np.exp(A) * dt, axis=0)
    want = D[:, None] * v
    for t in range(T):
        for j in range(t + 1):
            want[t] = want[t] + (np.exp(s[t] - s[j]) * dt[j] * (Cc[t, 0] @ B[j, 0]))[:, None] * v[j]
    assert np.allclose(got, want)


def test_oracle_shared_weights_and_missing_feed_forward():
    cfg = PM.config([PM.gla(ff=None), PM.mamba2(), PM.gla(ff=None, weights_of=0)], width=64, vocab=40)
    w = PM.weights(cfg, 5)
    assert not any(n.startswith("l2.") or n.startswith("l0.mlp") for n in w)
    t = [3, 1, 4, 1, 5]
    full, hidden = O.forward(cfg, w, t, return_layers=True)
    w2 = dict(w, **{"l2" + n[2:]: a for n, a in w.items() if n.startswith("l0.")})
    cfg2 = dict(cfg, layers=[cfg["layers"][0], cfg["layers"][1], PM.gla(ff=None)])
    assert np.array_equal(full, O.forward(cfg2, w2, t)) and hidden.shape == (3, 5, 64)


@pytest.mark.parametrize("taps", [1, 2, 4])
def test_oracle_convolution(taps):
    g = np.random.default_rng(taps)
    x, w, b = g.standard_normal((6, 3)), g.standard_normal((3, taps)), g.standard_normal(3)
    y = O.causal_conv(x, w, b)
    for t in range(6):
        want = b + sum(w[:, taps - 1 - j] * x[t - j] for j in range(taps) if t - j >= 0)
        assert np.allclose(y[t], want)
