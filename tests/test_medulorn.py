"""The Medulorn design on the CPU: both readers of its config.json, what they and the library refuse, and the plain restatement
(medulorn_oracle.py) against properties it must have."""
import ctypes as C
import json

import numpy as np
import pytest

import medulorn_models as MM
import medulorn_oracle as O
from layered_helpers import same_fields


def raw_config():
    return MM.config([MM.attention(), MM.parallel(mlp=MM.moe()), MM.attention(heads=3, kv_heads=3, chunk=None, turn=MM.rot(12), mlp=None),
                      MM.parallel(window=None, turn=MM.rot(24, 300.0), decay=[0.0, 0.5, 1.0], mlp=MM.moe(experts=5, top=2, shared=None)), MM.attention(turn=None, mlp=MM.moe(top=1))],
                     width=144, vocab=211, eps=3e-6, alpha=2.25, scale=7.5, cap=None)


def test_readers_agree(pkg, tmp_path):
    L, raw = pkg._lib, raw_config()
    p = tmp_path / "config.json"
    p.write_text(json.dumps(raw))
    c = L.ModelConfigC()
    L.check(L.lib().nvl_load_config_json(str(p).encode(), C.byref(c)))
    want = pkg.config.load_model_config(raw)
    assert (c.vocab_size, c.hidden, c.num_layers, c.max_seq_len, c.token_shift) == (211, 144, 5, 4096, 1) == \
        (want.vocab_size, want.hidden, want.num_layers, want.max_seq_len, want.token_shift)
    assert abs(c.norm_eps - 3e-6) < 1e-12 and c.norm_type == L.NORM[want.norm_type] == 2 and c.position_type == L.POS[want.position_type] == 2
    assert c.activation_type == L.ACT[want.activation_type] == 5 and c.block_style == L.BLOCK[want.block_style] == 4
    assert c.stream_scale == want.stream_scale == 2.25 and c.embedding_multiplier == want.embedding_multiplier == 7.5 and c.logit_softcap == want.logit_softcap == 0.0
    n = L.lib().nvl_load_layers_json(str(p).encode(), None, 0)
    arr = (L.LayerConfigC * n)()
    assert L.lib().nvl_load_layers_json(str(p).encode(), arr, n) == n == len(want.layers) == 5
    for a, w in zip(arr, want.layers):
        same_fields(L, a, w)
    assert [(a.chunk, a.window, a.keep_first) for a in arr] == [(50, 0, 0), (0, 30, 3), (0, 0, 0), (0, 0, 0), (50, 0, 0)]
    assert [(a.qk_norm, a.sink, a.qkv_bias, a.mixer2, a.rot_dim) for a in arr] == [(1, 1, 1, 0, 40), (2, 2, 0, 5, 16), (1, 1, 1, 0, 12), (2, 2, 0, 5, 24), (1, 1, 1, 0, 0)]
    assert [(a.rot_factor, a.rot_low, a.rot_high, a.rot_original) for a in arr[:2]] == [(0, 0, 0, 0), (8, 1, 4, 60)]
    assert [(a.experts, a.top_k, a.expert_dim, a.expert_limit, a.ffn_dim, a.ffn_act, a.ffn_limit) for a in arr] == \
        [(0, 0, 0, 0, 88, 0, 0), (10, 3, 40, 1.5, 56, 3, 2.5), (0, 0, 0, 0, 0, 0, 0), (5, 2, 40, 1.5, 0, 0, 0), (10, 1, 40, 1.5, 56, 3, 2.5)]
    assert list(arr[3].decay[:4]) == [0.0, 0.5, 1.0, 0.0] and (arr[1].heads2, arr[1].dim2, arr[1].vdim2) == (3, 20, 28)


def test_readers_refuse_what_they_do_not_know(pkg, tmp_path):
    L = pkg._lib
    p = tmp_path / "config.json"
    a, b = MM.attention(), MM.parallel()
    drop = lambda ly, *ks: dict(ly, mixer={n: v for n, v in ly["mixer"].items() if n not in ks})
    inner = lambda side, **kw: dict(b, mixer=dict(b["mixer"], **{side: dict(b["mixer"][side], **kw)}))
    moe = MM.moe()
    for layers in ([], [dict(a, type="gla")], [dict(a, mlp=dict(kind="hashed", ff=8))], [drop(a, "kv_heads")], [drop(a, "scale")], [drop(b, "right")], [drop(b, "left_scale")],
                   [inner("right", decay=[0.5])], [inner("right", decay=[0.5, "x", 0.1])], [dict(a, mlp=dict(moe, expert=dict(ff=8)))], [dict(a, mlp=dict(moe, shared=dict(ff=8)))],
                   [MM.parallel(turn=dict(base=1e4, dims=16, scaling=dict(factor=2.0, low=1.0, original=50)))]):
        raw = MM.config(layers)
        p.write_text(json.dumps(raw))
        assert L.lib().nvl_load_config_json(str(p).encode(), C.byref(L.ModelConfigC())) == -1, layers
        if layers:
            with pytest.raises((KeyError, ValueError)):
                pkg.config.load_model_config(raw)
    for key in ("postln_alpha", "embedding"):
        p.write_text(json.dumps({k: v for k, v in MM.config([a]).items() if k != key}))
        assert L.lib().nvl_load_config_json(str(p).encode(), C.byref(L.ModelConfigC())) == -1


def test_create_refuses_bad_lists_before_touching_a_device(pkg):
    L = pkg._lib
    from importlib import import_module
    M = import_module("nano-vllm-go_amd.model")
    opts = L.RuntimeOptsC(device=0, precision=0, max_seqs=2, tp_size=1)
    h = C.c_void_p()

    def create(raw, layer=None, **over):
        cfg = dict(pkg.config.load_model_config(raw).to_dict(), **over)
        if layer:
            cfg["layers"][0].update(layer)
        return L.lib().nvl_create_layers(C.byref(M._cfg_struct(cfg)), M._layer_structs(cfg["layers"]), C.byref(opts), C.byref(h))
    for layers in ([MM.attention(heads=5)], [MM.attention(kv_heads=0)], [MM.attention(dim=0, turn=None)], [MM.attention(turn=MM.rot(42))], [MM.attention(turn=MM.rot(7))],
                   [MM.parallel(keep=-1)], [MM.parallel(decay=[0.5, 1.5, 0.1])], [MM.parallel(decay=[0.5, -0.5, 0.1])], [MM.parallel(heads2=0, decay=[])],
                   [MM.parallel(turn=MM.rot(16, 1e4, (2.0, 4.0, 1.0, 50)))], [MM.parallel(turn=MM.rot(16, 1.0))], [MM.attention(mlp=MM.moe(top=11))],
                   [MM.attention(mlp=MM.moe(experts=300))], [MM.attention(mlp=MM.moe(shared_limit=0.0))]):
        try:
            assert create(MM.config(layers)) == -1, layers
        except (KeyError, ValueError):
            pass
    good = MM.config([MM.attention()])
    for over in (dict(window=9), dict(keep_first=2), dict(ungated=0), dict(mixer2=3), dict(qk_norm=3), dict(sink=5), dict(mixer="gla")):
        assert create(good, over) == -1, over
    assert create(good, activation_type="geglu") == -1 and create(good, block_style="sandwich") == -1 and create(good, stream_scale=0.0) == -1
    assert create(good, norm_type="layernorm") == -1 and create(good, side_dim=8) == -1
    if L.lib().nvl_device_count() == 0:
        assert create(raw_config()) == -8                                    # fine until the device is asked for


def test_synthetic_shapes_cover_the_checkpoint(pkg):
    """synth.layered_shapes names every tensor of the design: as many numbers as a checkpoint of the same configuration."""
    raw = raw_config()
    cfg = pkg.config.load_model_config(raw).to_dict()
    assert sum(int(np.prod(s)) for _, _, s, _ in pkg.synth.layered_shapes(cfg)) == sum(a.size for a in MM.weights(raw, 0).values())


# ---- the plain restatement ----
def changed(cfg, w, at, n=40):
    t = np.random.default_rng(0).integers(0, cfg["vocab"], n)
    b = t.copy()
    b[at] = (b[at] + 1) % cfg["vocab"]
    return np.abs(O.forward(cfg, w, b) - O.forward(cfg, w, t)).max(axis=1)


def test_oracle_chunks_end_and_shift_reaches_one_token():
    cfg = MM.config([MM.attention(chunk=8)], width=96, vocab=50)
    w = MM.weights(cfg, 3)
    d = changed(cfg, w, 10)
    assert np.all(d[:10] == 0) and np.all(d[10:16] > 1e-9) and np.all(d[16:] == 0)
    d = changed(cfg, w, 15)                                                  # the last of its chunk: the next chunk's first key has its shift
    assert np.all(d[:15] == 0) and np.all(d[15:24] > 1e-9) and np.all(d[24:] == 0)


def test_oracle_windows_keep_the_first_tokens():
    cfg = MM.config([MM.parallel(window=6, keep=2, right_scale=0.0)], width=96, vocab=50)
    w = MM.weights(cfg, 4)
    w["l0.shift"] = np.zeros_like(w["l0.shift"])
    for at, last in ((1, 40), (2, 8), (9, 15)):
        d = changed(cfg, w, at)
        assert np.all(d[:at] == 0) and np.all(d[at:last] > 1e-12) and np.all(d[last:] == 0), at


def test_oracle_norms_and_sums():
    g = np.random.default_rng(1)
    x = 3.0 + g.standard_normal((4, 50))
    assert np.allclose((O.scalar_norm(x, 2.0, 0.0) ** 2).mean(axis=1), 4.0) and np.allclose(O.scalar_norm(x, 1.0, 1e9), 0.0, atol=1e-3)
    h = g.standard_normal((3, 5))
    mu = np.array([0.0, 1.0, 0.25, -1.0, 2.0])
    y = O.token_shift(h, mu)
    assert np.allclose(y[0], h[0] * (1 - mu)) and np.allclose(y[2], h[2] + (h[1] - h[2]) * mu) and np.allclose(y[1:, 1], h[:-1, 1])


def test_oracle_rotation():
    f = O.frequencies(dict(base=100.0, dims=4))
    assert np.allclose(f, [1.0, 0.1])
    x = np.zeros((4, 1, 5))
    x[:, 0, 0], x[:, 0, 4] = 1.0, 7.0
    y = O.rotated(x, dict(base=100.0, dims=4))[:, 0]
    assert np.allclose(y[:, 0], np.cos(np.arange(4))) and np.allclose(y[:, 2], np.sin(np.arange(4))) and np.allclose(y[:, 4], 7.0) and np.allclose(y[:, [1, 3]], 0)
    sc = dict(factor=8.0, low=1.0, high=4.0, original=100.0)
    base = (2 * np.pi / 50.0) ** -2.0                                         # dims 4: pair 1 has a wavelength of 50 tokens, pair 0 one of 2 pi
    f = O.frequencies(dict(base=base, dims=4, scaling=sc))
    s = (100.0 / 50.0 - 1.0) / 3.0
    assert np.allclose(f, [1.0, (2 * np.pi / 50.0) * ((1 - s) / 8.0 + s)])
    assert np.allclose(O.frequencies(dict(base=1e12, dims=4, scaling=sc)), [1.0, 1e-6 / 8.0])


def test_oracle_sinks():
    p = O.sink_softmax(np.array([[0.0, np.log(3.0)], [900.0, 900.0]]), np.array([0.0, 900.0 + np.log(2.0)]))
    assert np.allclose(p, [[0.2, 0.6], [0.25, 0.25]])


def test_oracle_lightning():
    g = np.random.default_rng(2)
    q, k, v = g.standard_normal((9, 2, 3)), g.standard_normal((9, 2, 3)), g.standard_normal((9, 2, 4))
    o = O.lightning(q, k, v, [0.5, 1.0])
    for h, d in ((0, 0.5), (1, 1.0)):
        for t in range(9):
            assert np.allclose(o[t, h], sum(d ** (t - s) * (q[t, h] @ k[s, h]) * v[s, h] for s in range(t + 1)))


def test_oracle_experts():
    z = np.array([0.1, 2.0, -1.0, 1.9, 0.5])
    order, p, gap = O.choose(z, 2)
    assert order.tolist() == [1, 3] and np.isclose(gap, 1.4) and np.allclose(p, np.exp([2.0, 1.9]) / np.exp([2.0, 1.9]).sum())
    one = {"e.gate": np.ones((1, 1)), "e.up": np.array([[2.0]]), "e.down": np.ones((1, 1))}
    x = np.array([[-3.0], [0.5], [4.0]])
    sg = lambda t: 1 / (1 + np.exp(-1.702 * t))
    assert np.allclose(O.clamped_glu(x, one, "e", 1.5)[:, 0], [-3 * sg(-3) * (1 - 1.5), 0.5 * sg(0.5) * 2.0, 1.5 * sg(1.5) * 2.5])
    w = dict(gate=np.ones((1, 1)), up=np.array([[2.0]]), down=np.ones((1, 1)))
    assert np.allclose(O.relu_glu(x, w)[:, 0], [0.0, 0.5, 32.0])
