"""The Lufazen design on the CPU: both readers of its config.json, what they and the library refuse, and the plain restatement
(lufazen_oracle.py) against properties it must have."""
import ctypes as C
import json

import numpy as np
import pytest

import lufazen_models as LM
import lufazen_oracle as O
from layered_helpers import same_fields


def both_kinds():
    return LM.config([LM.latent(), LM.delta(), LM.latent(kv_from=0, heads=5, scaling=None, rot=48, ff=None)], width=144, vocab=211, eps=3e-6, cap=9.5)


def all_shared():
    return LM.config([LM.latent(), LM.delta(ff=None), LM.latent(kv_from=0, heads=5, ff=64)], width=144, vocab=211, eps=3e-6, cap=9.5)


def test_readers_agree(pkg, tmp_path):
    L, raw = pkg._lib, all_shared()
    p = tmp_path / "config.json"
    p.write_text(json.dumps(raw))
    c = L.ModelConfigC()
    L.check(L.lib().nvl_load_config_json(str(p).encode(), C.byref(c)))
    want = pkg.config.load_model_config(raw)
    assert (c.vocab_size, c.hidden, c.num_layers, c.max_seq_len) == (211, 144, 3, 4096) == (want.vocab_size, want.hidden, want.num_layers, want.max_seq_len)
    assert abs(c.norm_eps - 3e-6) < 1e-12 and c.norm_weight_offset == 1.0 == want.norm_weight_offset and c.logit_softcap == 9.5 == want.logit_softcap
    assert c.activation_type == L.ACT[want.activation_type] == 3 and c.block_style == L.BLOCK[want.block_style] == 3
    n = L.lib().nvl_load_layers_json(str(p).encode(), None, 0)
    arr = (L.LayerConfigC * n)()
    assert L.lib().nvl_load_layers_json(str(p).encode(), arr, n) == n == len(want.layers) == 3
    for a, w in zip(arr, want.layers):
        same_fields(L, a, w)
    assert arr[2].kv_from == 0 and arr[0].kv_from == -1 and arr[1].ffn_dim == 0 and arr[0].rot_dim == 48 and arr[0].gate_per_head == 1
    assert (arr[0].rot_factor, arr[0].rot_original, arr[0].rot_fast, arr[0].rot_slow, arr[0].rot_base) == (3.0, 64.0, 8.0, 1.0, 1000.0)
    assert (arr[1].kv_heads, arr[1].conv_taps) == (2, 4) and abs(arr[0].ffn_limit - 1.1) < 1e-6


def test_readers_refuse_what_they_do_not_know(pkg, tmp_path):
    L = pkg._lib
    p = tmp_path / "config.json"
    lat, dl = LM.latent(), LM.delta()
    for layers in ([], [dict(dl, type="gla")], [dict(dl, mlp=dict(kind="experts", ff=8, limit=1.0))], [dict(dl, mlp=dict(kind="dense", ff=8))],
                   [dict(lat, mixer=dict(lat["mixer"], rot_dim=16))], [dict(lat, mixer={k: v for k, v in lat["mixer"].items() if k != "rot"})]):
        raw = dict(LM.config(layers))
        p.write_text(json.dumps(raw))
        c = L.ModelConfigC()
        assert L.lib().nvl_load_config_json(str(p).encode(), C.byref(c)) == -1, layers
        if layers:
            with pytest.raises((KeyError, ValueError)):
                pkg.config.load_model_config(raw)


def test_create_refuses_bad_lists_before_touching_a_device(pkg):
    L = pkg._lib
    from importlib import import_module
    M = import_module("nano-vllm-go_amd.model")
    opts = L.RuntimeOptsC(device=0, precision=0, max_seqs=2, tp_size=1)
    h = C.c_void_p()

    def create(raw):
        cfg = pkg.config.load_model_config(raw).to_dict()
        return L.lib().nvl_create_layers(C.byref(M._cfg_struct(cfg)), M._layer_structs(cfg["layers"]), C.byref(opts), C.byref(h))
    for layers in ([LM.latent(kv_from=0)], [LM.latent(), LM.latent(kv_from=2), LM.latent()], [LM.delta(), LM.latent(kv_from=0)],
                   [LM.latent(), LM.latent(kv_from=0), LM.latent(kv_from=1)], [LM.latent(), LM.latent(kv_from=0, kv_rank=80)],
                   [LM.latent(), LM.latent(kv_from=0, base=999.0)], [LM.latent(rot=33)], [LM.delta(heads=4, kv_heads=3)], [LM.delta(conv=0)],
                   [LM.delta(limit=0.0)], [LM.latent(scaling=(2.0, 0, 8.0, 1.0))], both_kinds()["layers"]):
        assert create(LM.config(layers)) == -1, layers
    assert create(LM.config([LM.delta()], cap=-1.0)) == -1
    if L.lib().nvl_device_count() == 0:
        assert create(all_shared()) == -8                                    # fine until the device is asked for
    cfg = pkg.config.load_model_config(all_shared()).to_dict()
    assert L.lib().nvl_create(C.byref(M._cfg_struct(cfg)), C.byref(opts), C.byref(h)) == -1          # needs its layer list


def test_synthetic_shapes_cover_the_checkpoint(pkg):
    """synth.layered_shapes names every tensor of the design: as many numbers as a checkpoint of the same configuration."""
    raw = all_shared()
    w = LM.weights(raw, 0, a_rank=8, g_rank=8)
    cfg = pkg.config.load_model_config(raw).to_dict()
    assert sum(int(np.prod(s)) for _, _, s, _ in pkg.synth.layered_shapes(cfg, decay_rank=8)) == sum(a.size for a in w.values())


# ---- the plain restatement ----
def test_oracle_is_causal_and_deep_history_matters():
    cfg = LM.config([LM.latent(), LM.delta()], width=96, vocab=50)
    w = LM.weights(cfg, 3, decay_bias=-4.0)
    t = np.random.default_rng(0).integers(0, 50, 30)
    a = O.forward(cfg, w, t)
    b = t.copy()
    b[10] = (b[10] + 1) % 50
    d = np.abs(O.forward(cfg, w, b) - a).max(axis=1)
    assert np.all(d[:10] == 0) and np.all(d[10:] > 1e-9)


def test_oracle_rotation():
    rot = LM.latent(rot=12)["mixer"]["rot"]
    g = np.random.default_rng(1)
    q, k = g.standard_normal(12), g.standard_normal(12)
    Q, K = O.rotate(np.tile(q, (9, 1)), rot), O.rotate(np.tile(k, (9, 1)), rot)
    mag = 0.1 * np.log(3.0) + 1.0
    s = Q @ K.T
    for off in range(-8, 9):
        assert np.ptp(np.diagonal(s, off)) < 1e-9                            # scores depend on the distance only
    assert np.isclose(s[0, 0], q @ k * mag ** 2) and not np.isclose(s[1, 0], s[0, 0]) and not np.isclose(s[1, 0], s[0, 1])
    f, m = O.frequencies(dict(dims=64, base=1000.0, scaling=dict(factor=4.0, original=512, fast=32.0, slow=1.0)))
    plain, one = O.frequencies(dict(dims=64, base=1000.0, scaling=None))
    r = f / plain
    assert one == 1.0 and m > 1.0 and np.allclose(r[:3], 1.0) and np.isclose(r[-1], 0.25) and np.all(np.diff(r) <= 1e-12) and np.any((r > 0.3) & (r < 0.95))


def test_oracle_delta_rule():
    g = np.random.default_rng(2)
    T, H, d, dv = 12, 2, 5, 3
    k, q, v = O.unit(g.standard_normal((T, H, d))), g.standard_normal((T, H, d)), g.standard_normal((T, H, dv))
    la, beta = -g.uniform(0, 1, (T, H, d)), g.uniform(0, 1, (T, H))
    # step size 1: what is written under a unit key is read back at once, whatever was there before
    assert np.allclose(O.delta_recurrence(k, k, v, la, np.ones((T, H))), v, atol=1e-5)
    # the same recurrence with explicit transition matrices
    o = O.delta_recurrence(q, k, v, la, beta)
    for h in range(H):
        S = np.zeros((d, dv))
        for t in range(T):
            S = (np.eye(d) - beta[t, h] * np.outer(k[t, h], k[t, h])) @ np.diag(np.exp(la[t, h])) @ S + beta[t, h] * np.outer(k[t, h], v[t, h])
            assert np.allclose(o[t, h], S.T @ q[t, h])


def test_oracle_shared_latents():
    """A layer that reads another layer's latents equals one with latents of its own made by the same tensors from the same input."""
    cfg = LM.config([LM.latent(ff=None), LM.latent(ff=None, kv_from=0)], width=64, vocab=40)
    w = LM.weights(cfg, 5)
    assert not any(n.startswith("l1.mix.dkv") for n in w)
    w["l0.ls1"] = np.zeros_like(w["l0.ls1"])                                 # layer 0 leaves the stream as it was
    own = dict(cfg, layers=[cfg["layers"][0], LM.latent(ff=None)])
    w2 = dict(w, **{"l1.mix.dkv": w["l0.mix.dkv"], "l1.mix.dkv.norm": w["l0.mix.dkv.norm"]})
    t = [3, 1, 4, 1, 5, 9, 2, 6]
    assert np.allclose(O.forward(cfg, w, t), O.forward(own, w2, t))


@pytest.mark.parametrize("taps", [1, 2, 5])
def test_oracle_convolution(taps):
    g = np.random.default_rng(taps)
    x, w = g.standard_normal((6, 3)), g.standard_normal((3, taps))
    y = O.causal_conv(x, w)
    for t in range(6):
        assert np.allclose(y[t], sum(w[:, taps - 1 - j] * x[t - j] for j in range(taps) if t - j >= 0))


def test_oracle_clamps_and_caps():
    one = np.ones((1, 1))
    x = np.array([[-9.0], [-0.5], [0.5], [9.0]])
    y = O.clamped_glu(x, one, one, one, 1.5)[:, 0]
    s = lambda z: 1 / (1 + np.exp(-1.702 * z))
    assert np.allclose(y, [-9 * s(-9) * (1 - 1.5), -0.5 * s(-0.5) * 0.5, 0.5 * s(0.5) * 1.5, 1.5 * s(1.5) * 2.5])
    cfg = LM.config([LM.delta()], width=48, vocab=30, cap=0.5)
    assert np.abs(O.forward(cfg, LM.weights(cfg, 1), [1, 2, 3])).max() <= 0.5
