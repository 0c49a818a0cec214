"""CPU checks of the Pemuvik design: configuration and tensor table of zig_gpt2_amd/lm.py, the registry, and the float64 oracle's
own consistency (portions against whole prompts, each mechanism on hand-made inputs)."""
import json
import math

import numpy as np
import pytest

import pemuvik_oracle as po
import pemuvik_testlib as pl
from zig_gpt2_amd import lm, models


def small_cfg():
    return pl.config([pl.attn_layer(v_mix=False, mlp=pl.dense()), pl.attn_layer(heads=6, mlp=pl.moe()), pl.latent_layer(mlp=pl.moe(identity=0, groups=None, shared=0)),
                      pl.attn_layer(size=0, mlp=None), pl.latent_layer(heads=2, vdim=5, mlp=pl.dense(ff=9))])


def test_configuration_round_trip_and_tensor_table():
    cfg = small_cfg()
    c = lm.LMConfig.from_json(cfg)
    assert c.architecture == "Pemuvik" and c.tied_head
    assert [l.mixer for l in c.layers] == ["rotary_attention", "rotary_attention", "latent_attention", "rotary_attention", "latent_attention"]
    assert lm.LMConfig.from_json(json.loads(json.dumps(c.to_json()))) == c and c.to_json() == cfg
    assert [l.window for l in c.layers] == [9, 9, 0, 0, 0] and all(l.chunk == 0 and not l.rot_halves for l in c.layers)
    assert [l.value_mix for l in c.layers] == [False, True, False, True, False] and c.layers[2].sink and not c.layers[2].head_gate and c.layers[2].q_rank == 0
    assert c.layers[1].identity == 2 and c.layers[1].route_groups == 4 and c.layers[1].route_keep == 2 and c.layers[1].shared_gate
    assert c.layers[2].identity == 0 and c.layers[2].route_groups == 1 and c.layers[2].shared_width == 0
    t = c.tensor_shapes()
    assert t["l0.mix.q"] == (48, 40) and t["l0.mix.q.b"] == (48,) and t["l0.mix.k.b"] == (24,) and t["l0.mix.v.b"] == (16,) and t["l0.mix.o.b"] == (40,)
    assert t["l0.mix.pb"] == (4,) and "l0.mix.vmix" not in t and t["l1.mix.vmix"] == () and t["l1.mix.o"] == (40, 48)
    assert t["l0.mlp.gate"] == (28, 40) and t["l0.mlp.up"] == (28, 40) and t["l0.mlp.down"] == (40, 28)
    assert t["l1.mlp.router"] == (8, 40) and t["l1.mlp.correction"] == (8,) and "l1.mlp.e6.up" not in t and t["l1.mlp.shared.sg"] == (1, 40)
    assert t["l2.mlp.router"] == (6, 40) and "l2.mlp.shared.up" not in t
    assert t["l2.mix.sink"] == (3,) and t["l2.mix.q"] == (48, 40) and t["l2.mix.dkv"] == (26, 40) and "l2.mix.g" not in t and "l2.mix.q.b" not in t
    assert t["l3.ls1"] == (40,) and "l3.ls2" not in t and "l3.norm2" not in t and t["l4.ls2"] == (40,)
    assert "head" not in t and "l0.norm1b" not in t and "l0.norm2b" not in t and "l0.shift" not in t
    assert c.flags() == lm._lib.LM_SIDE_BY_SIDE | lm._lib.LM_LAYER_SCALE | lm._lib.LM_TIED_HEAD
    z = c.layers[1].to_c()
    assert (z.window, z.chunk, z.proj_bias, z.value_norm, z.value_mix, z.sigmoid_weights, z.sink, z.identity, z.shared_gate) == (9, 0, 1, 1, 1, 1, 0, 2, 1)
    assert "Pemuvik" in models.ARCHITECTURES


def test_other_designs_keep_their_masks_gates_and_routers():
    att = {"type": "attention", "mixer": {"heads": 2, "dim": 4, "vdim": 4, "scale": 0.5, "mask": {"size": 7}}, "mlp": {"kind": "dense", "ff": 8}}
    spec = lm.LayerSpec.from_json(att, "Duvulix")
    assert (spec.chunk, spec.window, spec.dense_act) == (7, 0, "polynorm") and not spec.sigmoid_weights and not spec.proj_bias and not spec.value_norm
    lat = {"type": "latent_attention", "mixer": pl.latent_layer()["mixer"], "mlp": None}
    spec = lm.LayerSpec.from_json(lat, "Duvulix")
    assert spec.head_gate and not spec.sink
    with pytest.raises(ValueError):
        lm.LayerSpec.from_json({"type": "mamba2", "mixer": {}, "mlp": None}, "Pemuvik")


def test_oracle_portions_equal_whole_prompts():
    cfg = small_cfg()
    w = pl.weights(cfg, seed=1)
    toks = pl.tokens(1, 40, cfg["vocab"])
    tr = []
    ref = po.forward(w, cfg, toks, trace=tr)
    assert len(tr) == 5 and tr[0].shape == (40, 40)
    for cuts in ([1, 2, 3, 17, 19], [10, 30], list(range(1, 40))):
        seq, rows, lo = po.Sequence(cfg), [], 0
        for hi in cuts + [40]:
            rows.append(po.forward(w, cfg, toks[lo:hi], seq))
            lo = hi
        assert np.abs(np.concatenate(rows) - ref).max() < 1e-9
    assert po.generate(w, cfg, toks[:5], 4) == po.generate(w, cfg, toks[:5], 6)[:4]


def test_rotation_and_window_on_hand_made_inputs():
    rot = {"base": 100.0, "dims": 4}
    v = np.array([[1.0, 2.0, 0.0, 3.0, 7.0]])
    r = po.rotate(v, [3], rot)  # pairs (0, 1) and (2, 3); the fifth channel passes
    want = [math.cos(3.0) - 2 * math.sin(3.0), 2 * math.cos(3.0) + math.sin(3.0), -3 * math.sin(0.3), 3 * math.cos(0.3), 7.0]
    assert np.allclose(r[0], want)
    q, k = np.random.default_rng(0).normal(size=(2, 1, 5))
    a = (po.rotate(q, [11], rot) * po.rotate(k, [4], rot)).sum()  # scores depend on the distance alone
    assert abs(a - (po.rotate(q, [107], rot) * po.rotate(k, [100], rot)).sum()) < 1e-9
    seen = po.window_visible([0, 2, 5], np.arange(6), {"size": 3})
    assert [np.flatnonzero(x).tolist() for x in seen] == [[0], [0, 1, 2], [3, 4, 5]]
    assert po.window_visible([4], np.arange(6), None).sum() == 5


def test_sinks_values_and_units_on_hand_made_inputs():
    s = np.array([[[0.0, math.log(3.0), -np.inf]]])
    assert np.allclose(po.sink_softmax(s, np.array([math.log(4.0)]))[0, 0], [1 / 8, 3 / 8, 0.0])
    assert np.allclose(po.sink_softmax(s, np.array([900.0]))[0, 0], 0.0) and np.allclose(po.sink_softmax(s, np.array([-900.0]))[0, 0], [0.25, 0.75, 0.0])
    assert np.allclose(po.unit(np.array([3.0, 4.0]), 0.0), np.array([3.0, 4.0]) / math.sqrt(12.5))
    assert np.allclose(po.mix_values(np.array([1.0]), 0.25, np.array([5.0])), 2.0)
    z = np.array([-2.0, 0.0, 1.5])
    exact = np.array([0.5 * v * (1.0 + math.erf(v / math.sqrt(2.0))) for v in z])
    assert np.abs(po.gelu_tanh(z) - exact).max() < 1e-3 and not np.allclose(po.gelu_tanh(z), exact, atol=1e-9)
    w = {"down": np.array([[2.0]]), "gate": np.array([[1.0]]), "up": np.array([[3.0]])}
    assert np.allclose(po.gated_unit(w, "", np.array([[0.5]]), po.silu), 2.0 * (0.5 / (1 + math.exp(-0.5))) * 1.5)


def test_router_on_hand_made_scores():
    z = np.log(np.array([[8.0, 1.0, 1.0, 4.0, 3.0, 3.0]]))  # softmax: 0.4 0.05 0.05 0.2 0.15 0.15
    pick, wt = po.route(z, np.zeros(6), 3, None)
    assert pick.tolist() == [[0, 3, 4]] and np.allclose(wt, np.array([0.4, 0.2, 0.15]) / 0.75)
    # groups rank by their largest score: {0.4, 0.05}, {0.05, 0.2}, {0.15, 0.15}; the sum of two would order them alike, so lift one
    assert po.route(z, np.zeros(6), 2, {"count": 3, "keep": 1})[0].tolist() == [[0, 1]]
    pick, wt = po.route(z, np.array([-0.5, 0, 0, 0, 0, 0]), 2, {"count": 3, "keep": 1})  # the second group's 0.2 beats 0.15 + 0.15
    assert pick.tolist() == [[3, 2]] and np.allclose(wt, [[0.8, 0.2]])
    # choice scores may be negative: what a dropped group holds must not come back as zero
    pick, wt = po.route(z, np.array([-0.5, -0.5, -0.5, -0.4, -0.9, -0.9]), 4, {"count": 3, "keep": 2})
    assert sorted(pick[0].tolist()) == [0, 1, 2, 3] and abs(wt.sum() - 1.0) < 1e-12


def test_pass_through_outputs_return_the_input():
    cfg = pl.config([pl.latent_layer(mlp=pl.moe(experts=2, identity=2, groups=None, top=1, shared=0))])
    w = pl.weights(cfg, seed=3)
    w["l0.mlp.correction"] = np.array([0.0, 0.0, 5.0, 0.0], np.float32)
    u = np.random.default_rng(3).normal(size=(4, 40))
    assert np.allclose(po.experts(w, "l0.mlp.", cfg["layers"][0]["mlp"], u), u)
