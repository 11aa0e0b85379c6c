"""The Bolinex design on the CPU: both readers of its config.json, what they and the library refuse, and the plain restatement
(bolinex_oracle.py) against properties it must have."""
import ctypes as C
import json

import numpy as np
import pytest

import bolinex_models as BM
import bolinex_oracle as O
from layered_helpers import same_fields


def raw_config():
    return BM.config([BM.attention(), BM.attention(heads=4, kv_heads=4, v_mix=False, window=None, cap=None, mlp=BM.moe()), BM.attention(mlp=None),
                      BM.attention(v_mix=False, mlp=BM.moe(experts=5, top=2, groups=None, shared=None))], width=144, vocab=211, eps=3e-6, side=18, positions=90)


def test_readers_agree(pkg, tmp_path):
    L, raw = pkg._lib, raw_config()
    p = tmp_path / "config.json"
    p.write_text(json.dumps(raw))
    c = L.ModelConfigC()
    L.check(L.lib().nvl_load_config_json(str(p).encode(), C.byref(c)))
    want = pkg.config.load_model_config(raw)
    assert (c.vocab_size, c.hidden, c.num_layers, c.max_seq_len, c.side_dim) == (211, 144, 4, 90, 18) == \
        (want.vocab_size, want.hidden, want.num_layers, want.max_seq_len, want.side_dim)
    assert abs(c.norm_eps - 3e-6) < 1e-12 and c.norm_type == L.NORM[want.norm_type] == 0 and c.position_type == L.POS[want.position_type] == 0
    assert c.activation_type == L.ACT[want.activation_type] == 4 and c.block_style == L.BLOCK[want.block_style] == 1
    n = L.lib().nvl_load_layers_json(str(p).encode(), None, 0)
    arr = (L.LayerConfigC * n)()
    assert L.lib().nvl_load_layers_json(str(p).encode(), arr, n) == n == len(want.layers) == 4
    for a, w in zip(arr, want.layers):
        same_fields(L, a, w)
    assert [a.v_mix for a in arr] == [1, 0, 1, 0] and [a.window for a in arr] == [50, 0, 50, 50] and [a.softcap for a in arr] == [9.0, 0.0, 9.0, 9.0]
    assert [(a.experts, a.top_k, a.expert_dim, a.expert_groups, a.groups_kept, a.ffn_dim, a.ffn_act) for a in arr] == \
        [(0, 0, 0, 0, 0, 88, 0), (12, 3, 40, 4, 2, 56, 1), (0, 0, 0, 0, 0, 0, 0), (5, 2, 40, 1, 1, 0, 1)]


def test_readers_refuse_what_they_do_not_know(pkg, tmp_path):
    L = pkg._lib
    p = tmp_path / "config.json"
    a = BM.attention()
    drop = lambda k: dict(a, mixer={n: v for n, v in a["mixer"].items() if n != k})
    for layers in ([], [dict(a, type="gla")], [dict(a, mlp=dict(kind="hashed", ff=8))], [drop("kv_heads")], [drop("scale")], [dict(a, mlp=dict(kind="moe", router=dict(experts=4, top=2)))]):
        raw = BM.config(layers)
        p.write_text(json.dumps(raw))
        c = L.ModelConfigC()
        assert L.lib().nvl_load_config_json(str(p).encode(), C.byref(c)) == -1, layers
        if layers:
            with pytest.raises((KeyError, ValueError)):
                pkg.config.load_model_config(raw)
    p.write_text(json.dumps({k: v for k, v in BM.config([a]).items() if k != "max_positions"}))
    assert L.lib().nvl_load_config_json(str(p).encode(), C.byref(L.ModelConfigC())) == -1


def test_create_refuses_bad_lists_before_touching_a_device(pkg):
    L = pkg._lib
    from importlib import import_module
    M = import_module("nano-vllm-go_amd.model")
    opts = L.RuntimeOptsC(device=0, precision=0, max_seqs=2, tp_size=1)
    h = C.c_void_p()

    def create(raw, **over):
        cfg = dict(pkg.config.load_model_config(raw).to_dict(), **over)
        return L.lib().nvl_create_layers(C.byref(M._cfg_struct(cfg)), M._layer_structs(cfg["layers"]), C.byref(opts), C.byref(h))
    for layers in ([BM.attention(heads=5, kv_heads=2)], [BM.attention(kv_heads=0)], [BM.attention(dim=0)], [BM.attention(), BM.attention(vdim=32)],
                   [BM.attention(mlp=BM.moe(experts=10, groups=(4, 2)))], [BM.attention(mlp=BM.moe(top=7))], [BM.attention(mlp=BM.moe(groups=(4, 5)))],
                   [BM.attention(mlp=BM.moe(experts=300, groups=None))]):
        assert create(BM.config(layers)) == -1, layers
    good = BM.config([BM.attention()])
    assert create(good, activation_type="geglu") == -1 and create(good, block_style="sandwich") == -1 and create(good, side_dim=-1) == -1
    assert create(good, norm_weight_offset=1.0) == -1
    if L.lib().nvl_device_count() == 0:
        assert create(raw_config()) == -8                                    # fine until the device is asked for


def test_synthetic_shapes_cover_the_checkpoint(pkg):
    """synth.layered_shapes names every tensor of the design: as many numbers as a checkpoint of the same configuration."""
    raw = raw_config()
    cfg = pkg.config.load_model_config(raw).to_dict()
    assert sum(int(np.prod(s)) for _, _, s, _ in pkg.synth.layered_shapes(cfg)) == sum(a.size for a in BM.weights(raw, 0).values())


# ---- the plain restatement ----
def test_oracle_is_causal_and_windows_end():
    cfg = BM.config([BM.attention(window=8), BM.attention(window=5, mlp=BM.moe())], width=96, vocab=50)
    w = BM.weights(cfg, 3)
    t = np.random.default_rng(0).integers(0, 50, 40)
    b = t.copy()
    b[10] = (b[10] + 1) % 50
    d = np.abs(O.forward(cfg, w, b) - O.forward(cfg, w, t)).max(axis=1)
    assert np.all(d[:10] == 0) and np.all(d[10:10 + 8 + 5 - 1] > 1e-9) and np.all(d[10 + 8 + 5 - 1:] == 0)


def test_oracle_norms():
    g = np.random.default_rng(1)
    x = 3.0 + g.standard_normal((4, 50))
    w, b = g.standard_normal(50), g.standard_normal(50)
    y = (O.layer_norm(x, w, b, 0.0) - b) / w
    assert np.allclose(y.mean(axis=1), 0) and np.allclose(y.std(axis=1), 1)
    assert np.allclose(O.layer_norm(x, w, b, 1e9), b, atol=1e-3)             # eps belongs under the root, with the variance
    assert np.allclose((O.rms_norm(x, w, 0.0) / w)[0], x[0] / np.sqrt((x[0] ** 2).mean()))


def test_oracle_scores():
    assert np.allclose(O.capped(np.array([1e-3, 1e6, -1e6]), 7.0), [1e-3, 7.0, -7.0], atol=1e-6) and O.capped(123.0, None) == 123.0
    b = O.distance_bias(np.array([2.0, 0.0]), np.array([0.5, 0.5]), np.array([0, 2, 6]))
    assert np.allclose(b, [[0, 2 * np.log(2), 2 * np.log(4)], [0, 0, 0]])
    # the bias is taken off after the cap: with equal keys the weights are (1 + r2 distance)^-r1
    mx = dict(heads=1, kv_heads=1, scale=1.0, softcap=0.1, mask=None)
    q, k = np.full((5, 1, 3), 9.0), np.ones((5, 1, 3))
    v = np.eye(5)[:, None]
    p = O.grouped_attention(q, k, v, mx, np.array([1.5]), np.array([0.3]))[4, 0]
    want = (1 + 0.3 * np.arange(4, -1, -1)) ** -1.5
    assert np.allclose(p, want / want.sum())


def test_oracle_groups_and_experts():
    ch = np.array([-0.9, -0.8, -0.1, -3.0, -0.5, -0.55, -2.0, -0.2])          # four pairs: -1.7, -3.1, -1.05, -2.2
    r = dict(experts=8, top=3, groups=dict(count=4, keep=2))
    order, gap = O.choose(ch, r)
    assert order.tolist() == [4, 5, 1] and np.isclose(gap, 0.1)               # not 2 or 7, the largest of all: their groups are out
    order, gap = O.choose(ch, dict(experts=8, top=2, groups=None))
    assert order.tolist() == [2, 7] and np.isclose(gap, 0.3)
    # weights are the scores without the correction, not renormalized
    g = np.random.default_rng(4)
    w = {f"e{e}.{n}": g.standard_normal((6, 6)) for e in range(8) for n in ("gate", "up", "down")}
    w.update(router=g.standard_normal((8, 6)), correction=np.array([9.0, 0, 0, 9.0, 0, 0, 0, 0]))
    h = g.standard_normal((3, 6))
    y = O.experts(h, w, dict(router=dict(experts=8, top=2, groups=None), shared=None))
    s = O.sigmoid(h @ w["router"].T)
    assert np.allclose(y, s[:, :1] * O.gated_ff(h, w, "e0") + s[:, 3:4] * O.gated_ff(h, w, "e3"))


def test_oracle_mixed_values():
    """The first mixing layer keeps its values; a later one with lambda 1 sees only those."""
    cfg = BM.config([BM.attention(v_mix=False, mlp=None), BM.attention(mlp=None), BM.attention(mlp=None)], width=64, vocab=40)
    w = BM.weights(cfg, 5)
    t = [3, 1, 4, 1, 5, 9, 2, 6]
    base = O.forward(cfg, w, t)
    assert np.array_equal(O.forward(cfg, dict(w, **{"l1.mix.vmix": np.float32(0.9)}), t), base)            # unused in the first
    w1 = dict(w, **{"l2.mix.vmix": np.float32(1.0)})
    assert np.allclose(O.forward(cfg, dict(w1, **{"l2.mix.v": w["l2.mix.v"] * 7}), t), O.forward(cfg, w1, t))
    assert np.abs(O.forward(cfg, w1, t) - base).max() > 1e-3


def test_oracle_activations():
    one = np.ones((1, 1))
    x = np.array([[-2.0], [0.5], [3.0]])
    assert np.allclose(O.squared_relu_ff(x, one, one)[:, 0], [0, 0.25, 9])
    assert np.allclose(O.gelu_tanh(np.array([0.0, 1.0, -1.0])), [0, 0.841192, -0.158808], atol=1e-5)
    w = dict(gate=np.eye(3), proj=np.eye(3), norm=np.ones(3))
    y = O.token_side(np.array([[1.0, 2.0, -1.0]]), np.array([[2.0, 0.0, 1.0]]), w, 0.0)
    z = np.array([2 * 0.841192, 0, -0.158808])
    assert np.allclose(y, z / np.sqrt((z ** 2).mean()), atol=1e-5)
