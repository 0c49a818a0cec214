"""CPU checks of the Duvulix design: configuration and tensor table of zig_gpt2_amd/lm.py, the registry, and the float64 oracle's
own consistency (portions against whole prompts, each mechanism on hand-made inputs)."""
import json
import math

import numpy as np
import pytest

import duvulix_oracle as do
import duvulix_testlib as dl
from zig_gpt2_amd import lm, models


def small_cfg():
    return dl.config([dl.mamba_layer(mlp=dl.dense()), dl.latent_layer(mlp=dl.dense()), dl.latent_layer(heads=2, vdim=5, kv_from=1, mlp=None),
                      dl.attn_layer(mlp=dl.dense(ff=9)), dl.mamba_layer(heads=3, vdim=7, groups=1, conv=1, norm_groups=3)])


def test_configuration_round_trip_and_tensor_table():
    cfg = small_cfg()
    c = lm.LMConfig.from_json(cfg)
    assert c.architecture == "Duvulix" and [l.mixer for l in c.layers] == ["ssd", "latent_attention", "latent_attention", "rotary_attention", "ssd"]
    assert lm.LMConfig.from_json(json.loads(json.dumps(c.to_json()))) == c and c.to_json() == cfg
    assert c.layers[0].dim == 12 and c.layers[0].kv_heads == 2 and c.layers[4].norm_groups == 3 and c.layers[4].conv == 1
    assert [l.kv_from for l in c.layers] == [None, None, 1, None, None] and c.layers[3].chunk == 9 and c.layers[1].q_rank == 0
    assert all(l.rot_halves for l in c.layers) and c.layers[1].head_gate and c.layers[0].dense_act == "polynorm"
    t = c.tensor_shapes()
    assert t["l0.mix.in"] == (2 * 40 + 2 * 2 * 12 + 4, 40) and t["l0.mix.conv"] == (88, 3) and t["l0.mix.conv.b"] == (88,) and t["l0.mix.norm"] == (40,)
    assert t["l0.mix.A_log"] == (4,) and t["l0.mix.D"] == (4,) and t["l0.mix.o"] == (40, 40) and t["l0.mlp.act"] == (4,)
    assert t["l1.mix.q"] == (48, 40) and t["l1.mix.dkv"] == (26, 40) and t["l1.mix.dkv.norm"] == (20,) and t["l1.mix.g"] == (3, 40)
    assert "l2.mix.dkv" not in t and "l2.mix.dkv.norm" not in t and t["l2.mix.uv"] == (10, 20) and "l2.norm2" not in t and "l1.mix.dq" not in t
    assert t["l3.mix.q"] == (48, 40) and t["l3.mix.k"] == (24, 40) and t["l3.mix.v"] == (16, 40) and t["l3.mix.o"] == (40, 32)
    assert "l0.shift" not in t and t["l0.norm1b"] == (40,) and t["head"] == (89, 40)
    assert c.flags() == lm._lib.LM_NO_SHIFT and c.layers[2].to_c().kv_from == 2 and c.layers[1].to_c().kv_from == 0
    assert "Duvulix" in models.ARCHITECTURES


def test_other_designs_keep_their_feed_forward_and_rotation():
    spec = lm.LayerSpec.from_json({"type": "hgrn2", "mixer": {"heads": 2, "dim": 4, "vdim": 4}, "mlp": {"kind": "dense", "ff": 8}}, "Tokosun")
    assert spec.dense_act == "relu2" and not spec.rot_halves and spec.to_c().dense_act == 0
    with pytest.raises(ValueError):
        lm.LayerSpec.from_json({"type": "hgrn2", "mixer": {"heads": 2, "dim": 4, "vdim": 4}, "mlp": None}, "Duvulix")


def test_oracle_portions_equal_whole_prompts():
    cfg = small_cfg()
    w = dl.weights(cfg, seed=1)
    toks = dl.tokens(1, 40, cfg["vocab"])
    tr = []
    ref = do.forward(w, cfg, toks, trace=tr)
    assert len(tr) == 5 and tr[0].shape == (40, 40)
    for cuts in ([1, 2, 3, 17, 19], [10, 30], list(range(1, 40))):
        seq, rows, lo = do.Sequence(cfg), [], 0
        for hi in cuts + [40]:
            rows.append(do.forward(w, cfg, toks[lo:hi], seq))
            lo = hi
        assert np.abs(np.concatenate(rows) - ref).max() < 1e-9
    assert do.generate(w, cfg, toks[:5], 4) == do.generate(w, cfg, toks[:5], 6)[:4]


def test_rotation_on_hand_made_vectors():
    rot = {"base": 100.0, "dims": 4}
    v = np.array([[1.0, 2.0, 0.0, 0.0, 7.0]])
    r = do.rotate(v, [3], rot)  # pairs (0, 2) and (1, 3); the fifth channel passes
    assert np.allclose(r[0], [math.cos(3.0), 2 * math.cos(0.3), math.sin(3.0), 2 * math.sin(0.3), 7.0])
    # scores depend on the distance alone
    q, k = np.random.default_rng(0).normal(size=(2, 1, 5))
    a = (do.rotate(q, [11], rot) * do.rotate(k, [4], rot)).sum()
    assert abs(a - (do.rotate(q, [107], rot) * do.rotate(k, [100], rot)).sum()) < 1e-9
    # the blend: pairs that turn often keep their frequency, slow ones are divided by the factor
    f, amp = do.rotary_frequencies({"base": 30000.0, "dims": 64, "scaling": {"factor": 5.0, "original": 700, "fast": 20.0, "slow": 1.5}})
    g = 30000.0 ** (-2.0 * np.arange(32) / 64)
    assert np.allclose(f[0], g[0]) and np.allclose(f[-1], g[-1] / 5.0) and abs(amp - (0.1 * math.log(5.0) + 1.0)) < 1e-12
    assert ((f <= g + 1e-15) & (f >= g / 5.0 - 1e-15)).all()


def test_chunks_on_hand_made_positions():
    seen = do.chunk_visible([0, 2, 3, 5, 6], np.arange(7), {"size": 3})
    assert [np.flatnonzero(r).tolist() for r in seen] == [[0], [0, 1, 2], [3], [3, 4, 5], [6]]
    assert do.chunk_visible([4], np.arange(6), None).sum() == 5


def test_convolution_and_recurrence_on_hand_made_inputs():
    w, b = np.array([[10.0, 1.0, 100.0]]), np.array([0.5])
    out, tail = do.causal_conv(w, b, np.array([[1.0], [2.0], [3.0]]), None)
    assert np.allclose(out[:, 0], [100.5, 201.5, 312.5]) and np.allclose(tail[:, 0], [2.0, 3.0])
    out2, tail2 = do.causal_conv(w, b, np.array([[4.0]]), tail)
    assert np.allclose(out2[0], 10 * 2 + 3 + 400 + 0.5) and np.allclose(tail2[:, 0], [3.0, 4.0])
    x, B, C = np.ones((3, 1, 1)), np.ones((3, 1, 2)), np.ones((3, 1, 2))
    dt = np.array([[1.0], [2.0], [0.0]])
    y, S = do.ssd_recurrence(x, B, C, dt, np.array([math.log(0.5)]), np.array([3.0]), None)
    s1 = 1.0
    s2 = math.exp(-0.5 * 2.0) * s1 + 2.0
    assert np.allclose(y[:, 0, 0], [2 * s1 + 3, 2 * s2 + 3, 2 * s2 + 3]) and np.allclose(S[0, :, 0], s2)
    y2, _ = do.ssd_recurrence(x[2:], B[2:], C[2:], dt[2:], np.array([math.log(0.5)]), np.array([3.0]), do.ssd_recurrence(x[:2], B[:2], C[:2], dt[:2], np.array([math.log(0.5)]), np.array([3.0]), None)[1])
    assert np.allclose(y2[0], y[2])
    assert np.allclose(do.softplus(np.array([-800.0, 0.0, 800.0])), [0.0, math.log(2.0), 800.0])


def test_norms_and_activation_on_hand_made_rows():
    v = np.array([[3.0, 4.0, 30.0, 40.0]])
    assert np.allclose(do.part_norm(np.array([1.0, 1.0, 2.0, 2.0]), v, 2, 0.0)[0], np.array([3, 4, 6, 8]) / math.sqrt(12.5))
    assert np.allclose(do.offset_norm(np.zeros(2), np.array([[1.0, 7.0]]), 0.0)[0], [0.2, 1.4])
    z = np.array([[1.0, -2.0]])
    want = 0.5 * z / math.sqrt(2.5) + 0.25 * z ** 2 / math.sqrt(8.5) + 2.0 * z ** 3 / math.sqrt(32.5) - 1.0
    assert np.allclose(do.polynorm([0.5, 0.25, 2.0, -1.0], z, 0.0), want)
