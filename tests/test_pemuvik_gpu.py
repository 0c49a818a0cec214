"""The Pemuvik design on the layered-model tier (zig_gpt2_amd/lm.py) against the float64 oracle of tests/pemuvik_oracle.py: every
mechanism alone, whole prompts against portions and token-by-token decoding, ragged batches, slots and pages that go round, heavy
keys hundreds of tokens back and on both sides of a window's edge, sinks, value mixing and pass-through experts that show, other
sizes, and generation through the library's entry points, the scheduler, the host program and the trace replay."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import lm_testlib as tl
import pemuvik_oracle as po
import pemuvik_testlib as pl
from zig_gpt2_amd import lm, models, weights_io

pytestmark = pytest.mark.gpu


def make(cfg, w, dtype="float32", **kw):
    kw.setdefault("max_tokens", 512)
    kw.setdefault("max_seqs", 4)
    m = lm.LayeredLM(lm.LMConfig.from_json(cfg), dtype=dtype, **kw)
    m.load_weights(w)
    return m


def run_whole(m, toks, want=None, trace=False):
    s = m.open()
    out = m.step([(s, toks, list(range(len(toks))) if want is None else want)], trace=trace)
    m.close_seq(s)
    return out


def run_cut(m, toks, cuts):
    """Feed toks in portions that end at `cuts`; all logits."""
    s = m.open()
    rows, lo = [], 0
    for hi in list(cuts) + [len(toks)]:
        if hi > lo:
            rows.append(m.step([(s, toks[lo:hi], list(range(hi - lo)))]))
        lo = hi
    m.close_seq(s)
    return np.concatenate(rows)


SINGLE = {
    "latent": [pl.latent_layer()],
    "latent_one_head": [pl.latent_layer(heads=1, dim=3, vdim=5, rot_dim=2, kv_rank=9, scale=0.9)],
    "latent_wide": [pl.latent_layer(heads=2, kv_rank=340, rot_dim=20, dim=30, vdim=40)],  # beyond the tiled prompt attention
    "attention": [pl.attn_layer()],
    "attention_two_layers_mix": [pl.attn_layer(), pl.attn_layer(heads=2, dim=9, scale=0.7), pl.attn_layer(v_mix=False, kv_heads=4), pl.attn_layer()],
    "attention_mix_begins_late": [pl.attn_layer(v_mix=False), pl.latent_layer(), pl.attn_layer(), pl.attn_layer(heads=6, size=4)],
    "attention_own_keys": [pl.attn_layer(heads=3, kv_heads=3, dim=8, vdim=8, size=5), pl.attn_layer(heads=6, kv_heads=3, dim=4, vdim=8, rot_dims=4, size=0)],
    "attention_odd_sizes": [pl.attn_layer(heads=5, kv_heads=1, dim=7, vdim=3, rot_dims=4, size=16), pl.attn_layer(heads=7, kv_heads=1, dim=5, vdim=3, rot_dims=2)],
    "attention_window_of_one": [pl.attn_layer(size=1)],  # every token sees itself
    "attention_whole_context": [pl.attn_layer(size=0, rot_dims=0)],  # no window, no rotation
    "attention_middle_heads": [pl.attn_layer(heads=12, kv_heads=2, dim=96, vdim=100, scale=0.1, size=20), pl.attn_layer(heads=9, kv_heads=1, dim=72, vdim=65, v_mix=False)],
    "attention_wide_heads": [pl.attn_layer(heads=2, kv_heads=1, dim=150, vdim=200, scale=0.05, size=20)],
    "attention_beyond_the_fused_kernels": [pl.attn_layer(heads=2, kv_heads=1, dim=260, vdim=20, rot_dims=250, scale=0.05, size=20), pl.attn_layer(kv_heads=1, dim=10, vdim=20)],
    "ff": [pl.attn_layer(mlp=pl.dense())],
    "ff_narrow": [pl.attn_layer(mlp=pl.dense(ff=1)), pl.latent_layer(mlp=pl.dense(ff=7))],
    "ff_long_rows": [pl.attn_layer(mlp=pl.dense(ff=1700))],  # second products that split their rows over waves
    "experts": [pl.attn_layer(mlp=pl.moe())],
    "experts_one_group": [pl.latent_layer(mlp=pl.moe(groups=None))],
    "experts_no_pass_through": [pl.latent_layer(mlp=pl.moe(experts=8, identity=0, groups=(2, 1), top=2))],
    "experts_mostly_pass_through": [pl.latent_layer(mlp=pl.moe(experts=1, identity=5, groups=(3, 2), top=4, shared=0))],
    "experts_all_chosen": [pl.attn_layer(mlp=pl.moe(experts=3, identity=1, groups=(2, 2), top=4, shared=5))],
    "experts_groups_of_one": [pl.attn_layer(mlp=pl.moe(experts=5, identity=2, groups=(7, 3), top=2, ff=3, shared=1))],
    "experts_many": [pl.attn_layer(mlp=pl.moe(experts=120, identity=8, groups=(16, 5), top=11, ff=6, shared=33))],
    "experts_long_rows": [pl.latent_layer(mlp=pl.moe(ff=1600, shared=1590, experts=2, identity=2, groups=(2, 1), top=1))],
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(SINGLE))
def test_each_mechanism_alone(name, dtype):
    cfg = pl.config(SINGLE[name], width=50 if "one_head" in name else 40)
    w = pl.weights(cfg, seed=sum(map(ord, name)), router_std=2.0)
    toks = pl.tokens(1, 83 if "one_head" in name else 37, cfg["vocab"])
    ref_tr = []
    ref = po.forward(w, cfg, toks, trace=ref_tr)
    m = make(cfg, w, dtype)
    got, tr = run_whole(m, toks, trace=True)
    tl.assert_close(tr, np.stack(ref_tr), dtype, "residual stream")
    tl.assert_close(got, ref, dtype, "logits")
    # the same prompt token by token: the decode kernels on the cached keys, values and latents
    step = run_cut(m, toks, range(1, len(toks)))
    tl.assert_close(step, ref, dtype, "decoded")
    m.close()


def full_cfg(**kw):
    return pl.config([pl.attn_layer(mlp=pl.dense()), pl.attn_layer(heads=6, mlp=pl.moe()), pl.latent_layer(mlp=pl.moe(experts=5, identity=1, groups=(3, 2), top=2, shared=7)),
                      pl.attn_layer(heads=2, dim=9, size=14, mlp=None), pl.attn_layer(heads=3, kv_heads=3, dim=4, vdim=5, rot_dims=2, scale=0.7, size=21, v_mix=False, mlp=pl.dense(ff=13)),
                      pl.latent_layer(heads=1, kv_rank=7, rot_dim=4, mlp=None), pl.attn_layer(size=5, mlp=pl.moe(groups=None, identity=1))], **kw)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_portions_of_several_sizes(dtype):
    cfg = full_cfg()
    w = pl.weights(cfg, seed=5)
    toks = pl.tokens(2, 90, cfg["vocab"])
    ref = po.forward(w, cfg, toks)
    m = make(cfg, w, dtype, page_tokens=8)
    tl.assert_close(run_whole(m, toks), ref, dtype)
    for cuts in ([2, 4, 7, 15, 16, 24, 25, 57, 88], [1, 2, 3, 40, 41, 43], list(range(9, 90, 9)), list(range(2, 90, 2)), [64], [8, 10, 19, 27, 29, 41, 43]):
        tl.assert_close(run_cut(m, toks, cuts), ref, dtype, cuts)
    # portions longer than one pass of the library are cut inside the step
    m2 = make(cfg, w, dtype, max_step_tokens=16, page_tokens=8)
    tl.assert_close(run_whole(m2, toks), ref, dtype)
    tl.assert_close(run_cut(m2, toks, [33, 35]), ref, dtype)
    m.close()
    m2.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_unequal_requests_in_one_batch(dtype):
    cfg = full_cfg()
    w = pl.weights(cfg, seed=7)
    lens = [41, 3, 17, 1]
    prompts = [pl.tokens(10 + i, n, cfg["vocab"]) for i, n in enumerate(lens)]
    refs = [po.forward(w, cfg, p) for p in prompts]
    m = make(cfg, w, dtype, page_tokens=4)
    seqs = [m.open() for _ in prompts]
    first = [30, 2, 9, 1]
    got = m.step([(s, p[:k], list(range(k))) for s, p, k in zip(seqs, prompts, first)])
    off = 0
    for r, k in zip(refs, first):
        tl.assert_close(got[off:off + k], r[:k], dtype)
        off += k
    entries = [(s, p[k:], list(range(len(p) - k))) for s, p, k in zip(seqs, prompts, first) if len(p) > k]
    got = m.step(entries)
    off = 0
    for r, p, k in zip(refs, prompts, first):
        if len(p) > k:
            tl.assert_close(got[off:off + len(p) - k], r[k:], dtype)
            off += len(p) - k
    # lock-step decoding of three sequences at different positions against each alone
    more = [pl.tokens(20 + i, 6, cfg["vocab"]) for i in range(3)]
    alone = [po.forward(w, cfg, np.concatenate([prompts[i], more[i]]))[len(prompts[i]):] for i in range(3)]
    rows = [m.step([(seqs[i], [more[i][t]], [0]) for i in range(3)]) for t in range(6)]
    for i in range(3):
        tl.assert_close(np.stack([r[i] for r in rows]), alone[i], dtype, i)
    m.close()


def test_decode_batches_of_every_size():
    """One to eight sequences in lock step, every batch size on its own captured graph, each row against its sequence alone; then steps
    of few rows that mix decoded tokens with short portions."""
    cfg = full_cfg()
    w = pl.weights(cfg, seed=9)
    m = make(cfg, w, max_seqs=8, page_tokens=8)
    seqs = [pl.tokens(100 + i, 5 + 3 * i + 14, cfg["vocab"]) for i in range(8)]
    refs = [po.forward(w, cfg, t) for t in seqs]
    slots = [m.open() for _ in seqs]
    at = [5 + 3 * i for i in range(8)]
    m.step([(s, t[:k], []) for s, t, k in zip(slots, seqs, at)])
    for n in (1, 2, 3, 4, 5, 6, 7, 8):
        got = m.step([(slots[i], [seqs[i][at[i]]], [0]) for i in range(n)])
        for i in range(n):
            tl.assert_close(got[i], refs[i][at[i]], "float32", (n, i))
            at[i] += 1
    for counts in ([2, 1, 3], [1, 2], [4, 1, 1, 2]):
        got = m.step([(slots[i], seqs[i][at[i]:at[i] + c], list(range(c))) for i, c in enumerate(counts) if at[i] + c <= len(seqs[i])])
        off = 0
        for i, c in enumerate(counts):
            if at[i] + c <= len(seqs[i]):
                tl.assert_close(got[off:off + c], refs[i][at[i]:at[i] + c], "float32", (counts, i))
                off += c
                at[i] += c
    m.close()


def test_decode_batches_of_many_heads():
    """Eight rows of 90 heads, five to a key head: a workgroup of the decode kernel then takes four query heads of a key head (and the fifth
    alone) instead of one; heads of each of the kernel's sizes, decoded in lock step and in steps of two entries with two to four rows."""
    cfg = pl.config([pl.attn_layer(heads=90, kv_heads=18, dim=6, vdim=5, size=20, v_mix=False), pl.attn_layer(heads=65, kv_heads=13, dim=70, vdim=9, scale=0.1, size=0, v_mix=False),
                     pl.attn_layer(heads=70, kv_heads=10, dim=9, vdim=130, size=11, v_mix=False)], width=20)
    w = pl.weights(cfg, seed=25)
    m = make(cfg, w, max_seqs=8, page_tokens=8)
    seqs = [pl.tokens(120 + i, 12 + 5 * i + 8, cfg["vocab"]) for i in range(8)]
    refs = [po.forward(w, cfg, t) for t in seqs]
    slots = [m.open() for _ in seqs]
    at = [12 + 5 * i for i in range(8)]
    m.step([(s, t[:k], []) for s, t, k in zip(slots, seqs, at)])
    for counts in ([1] * 8, [1] * 8, [4, 4], [2, 3], [1] * 8):
        got = m.step([(slots[i], seqs[i][at[i]:at[i] + c], list(range(c))) for i, c in enumerate(counts) if at[i] + c <= len(seqs[i])])
        off = 0
        for i, c in enumerate(counts):
            if at[i] + c <= len(seqs[i]):
                tl.assert_close(got[off:off + c], refs[i][at[i]:at[i] + c], "float32", (counts, i))
                off += c
                at[i] += c
    m.close()


def test_slots_and_pages_are_reused():
    """Two slots and a cache of 96 tokens in pages of 4.  A closed sequence gives its pages and its slot back; the next one starts on pages
    that held other keys, values and latents."""
    cfg = full_cfg()
    w = pl.weights(cfg, seed=8)
    m = make(cfg, w, max_tokens=96, max_seqs=2, page_tokens=4)
    total = m.free_tokens()
    a, b, c = (pl.tokens(30 + i, n, cfg["vocab"]) for i, n in enumerate((50, 38, 44)))
    ra, rb, rc = (po.forward(w, cfg, t) for t in (a, b, c))
    for rnd in range(2):
        sa, sb = m.open(), m.open()
        with pytest.raises(Exception):
            m.open()  # both slots taken
        for lo in range(0, 30, 10):
            got = m.step([(sa, a[lo:lo + 10], list(range(10))), (sb, b[lo:lo + 10], [9])])
            tl.assert_close(got[:10], ra[lo:lo + 10], "float32", (rnd, lo))
            tl.assert_close(got[10], rb[lo + 9], "float32", (rnd, lo))
        assert total - m.free_tokens() == 2 * 32  # whole pages per sequence
        with pytest.raises(Exception):
            m.step([(sa, np.concatenate([a, a]), [])])  # more than the cache holds
        m.close_seq(sb)  # its slot and pages go to a new sequence that starts from nothing
        sc = m.open()
        got = m.step([(sc, c, list(range(44))), (sa, a[30:], list(range(20)))])
        tl.assert_close(got[:44], rc, "float32", rnd)
        tl.assert_close(got[44:], ra[30:], "float32", rnd)
        assert m.seq_len(sa) == 50 and m.seq_len(sc) == 44
        m.close_seq(sa)
        m.close_seq(sc)
        assert m.free_tokens() == total
    m.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_windowed_sequences_outgrow_the_cache(dtype):
    """A stack that looks back one window at most returns the pages behind it while the sequence runs: 300 tokens through a cache of 80, in
    portions and decoded, two sequences taking each other's pages (pages smaller than a tile of keys)."""
    cfg = pl.config([pl.attn_layer(size=12, mlp=pl.dense()), pl.attn_layer(heads=2, size=20, mlp=pl.moe())])
    w = pl.weights(cfg, seed=33)
    a, b = pl.tokens(34, 300, cfg["vocab"]), pl.tokens(35, 300, cfg["vocab"])
    ra, rb = po.forward(w, cfg, a), po.forward(w, cfg, b)
    m = make(cfg, w, dtype, max_tokens=80, max_seqs=2, page_tokens=4)
    total = m.free_tokens()
    sa, sb = m.open(), m.open()
    lo, ga, gb = 0, [], []
    for n in [7, 2, 12, 3, 1, 1, 9, 11, 2, 5] * 5 + [12] * 2 + [1] * 11:
        got = m.step([(sa, a[lo:lo + n], list(range(n))), (sb, b[lo:lo + n], list(range(n)))])
        ga.append(got[:n])
        gb.append(got[n:])
        if dtype == "float32":
            tl.assert_close(got[:n], ra[lo:lo + n], dtype, lo)
            tl.assert_close(got[n:], rb[lo:lo + n], dtype, lo)
        lo += n
    tl.assert_close(np.concatenate(ga), ra, dtype)
    tl.assert_close(np.concatenate(gb), rb, dtype)
    assert lo == 300 and total - m.free_tokens() <= 2 * 28
    m.close_seq(sa)
    m.close_seq(sb)
    assert m.free_tokens() == total
    m.close()


def test_general_attention_kernel(monkeypatch):
    """The one-workgroup-per-row form of the windowed attention (what heads beyond the fused kernels take), on prompts, portions and decoded
    tokens over several key tiles."""
    monkeypatch.setenv("ZGPT2_LM_WINDOW_GENERAL", "1")
    cfg = pl.config([pl.attn_layer(size=90), pl.attn_layer(heads=2, kv_heads=1, dim=70, vdim=16, scale=0.08, size=33, v_mix=False), pl.attn_layer(size=0)])
    w = pl.weights(cfg, seed=21)
    toks = pl.tokens(22, 200, cfg["vocab"])
    ref = po.forward(w, cfg, toks)
    for dtype in ("float32", "bfloat16"):
        m = make(cfg, w, dtype)
        tl.assert_close(run_whole(m, toks), ref, dtype)
        tl.assert_close(run_cut(m, toks, [3, 64, 65, 130] + list(range(180, 200))), ref, dtype)
        m.close()


def _probe(cfg, w, toks, kind):
    po.PROBE = []
    try:
        ref = po.forward(w, cfg, toks)
        att = [p[1] for p in po.PROBE if p[0] == kind]
    finally:
        po.PROBE = None
    return ref, att


def _input_duals(cfg, w, ids):
    """In the first layer the mixer's input depends on the token alone.  Column t of the result has a product of one with the input of
    token ids[t] and of zero with every other listed token's."""
    return np.linalg.pinv(po.norm(w["l0.norm1"], w["embed"].astype(np.float64)[ids], cfg["norm"]["eps"]))


def test_far_latents_among_hundreds():
    """One key is made to stand out: the latent of one token id gets a large component that no other token of the prompt has, one head's key
    projection reads it and that head's query of another token id asks for it.  It sits at position 5, its queries hundreds of tokens
    later — across pages, key tiles and the shares of a split row."""
    n, W, KR = 420, 32, 16
    cfg = pl.config([pl.latent_layer(heads=3, dim=12, vdim=6, rot_dim=6, kv_rank=KR, scale=0.5)], width=W)
    w = pl.weights(cfg, seed=19)
    rng = np.random.default_rng(19)
    ids = rng.permutation(cfg["vocab"])[:22]
    dual = _input_duals(cfg, w, ids)
    toks = rng.choice(ids[2:], n).astype(np.int32)
    queries = (230, 300, 301, 388, 419)
    toks[5], toks[list(queries)] = ids[0], ids[1]
    lat, d = rng.normal(0.0, 1.0, KR), rng.normal(0.0, 1.0, 12)
    dkv, uk, q = (w[k].astype(np.float64).copy() for k in ("l0.mix.dkv", "l0.mix.uk", "l0.mix.q"))
    dkv[:KR] += 30.0 * np.outer(lat, dual[:, 0])
    uk[12:24] += np.outer(d, lat) * 0.5  # head 1
    q[18:30] += 8.0 * np.outer(d, dual[:, 1])
    w["l0.mix.dkv"], w["l0.mix.uk"], w["l0.mix.q"] = (pl.round_bf16(a.astype(np.float32)) for a in (dkv, uk, q))
    ref, att = _probe(cfg, w, toks, "latent_attention")
    assert all(att[-1][1, i, 5] > 0.8 for i in queries), [att[-1][1, i, 5] for i in queries]
    gone = toks.copy()
    gone[5] = toks[6]
    assert tl.rel_err(po.forward(w, cfg, gone)[list(queries)], ref[list(queries)]) > 1e-2
    for dtype, tol in (("float32", 2e-4), ("bfloat16", 4e-2)):
        m = make(cfg, w, dtype, page_tokens=16)
        for got in (run_whole(m, toks), run_cut(m, toks, [4, 5, 6, 100, 229, 230, 231, 333] + list(range(380, n)))):
            assert tl.rel_err(got[list(queries)], ref[list(queries)]) < tol
            if dtype == "bfloat16":
                tl.assert_close(got, ref, dtype)
            else:
                assert tl.rel_err(got, ref) < tol
        m.close()


@pytest.mark.parametrize("sink", [-60.0, 0.0, 3.0, 40.0, 120.0])
def test_sinks_from_nothing_to_everything(sink):
    """A sink far below every score counts nothing, one far above takes the whole weight (its exponential alone would overflow); in the first
    tokens it outweighs the few keys there are.  Prompts on the tiled and the general kernel, decoding through split rows."""
    cfg = pl.config([pl.latent_layer(heads=3, scale=0.8)])
    w = pl.weights(cfg, seed=29)
    w["l0.mix.sink"] = np.array([sink, 0.5 * sink, -sink], np.float32)
    toks = pl.tokens(29, 180, cfg["vocab"])
    ref = po.forward(w, cfg, toks)
    if sink:
        w2 = dict(w)
        w2["l0.mix.sink"] = -w["l0.mix.sink"]
        assert tl.rel_err(po.forward(w2, cfg, toks), ref) > 1e-2
    for dtype in ("float32", "bfloat16"):
        m = make(cfg, w, dtype)
        tl.assert_close(run_whole(m, toks), ref, dtype)
        tl.assert_close(run_cut(m, toks, [1, 2, 3, 70, 72] + list(range(150, 180))), ref, dtype)
        m.close()


@pytest.mark.parametrize("size", [1, 2, 31, 32, 64, 100])
def test_heavy_keys_inside_and_outside_a_window(size):
    """One token id's key stands out for another's queries (a large negative offset keeps every other key's weight small).  Queries sit one
    token inside the window's far edge, on it and behind it, where the key must weigh nothing."""
    n, W, D = 2 * size + 60, 32, 16
    cfg = pl.config([pl.attn_layer(heads=4, kv_heads=2, dim=D, vdim=10, scale=0.4, size=size, rot_dims=4)], width=W)
    w = pl.weights(cfg, seed=size)
    w["l0.mix.pb"] = np.array([-1.0, -2.0, -1.0, -6.0], np.float32)
    rng = np.random.default_rng(size)
    ids = rng.permutation(cfg["vocab"])[:22]
    dual = _input_duals(cfg, w, ids)
    d = np.concatenate([np.zeros(4), rng.normal(0.0, 1.0, D - 4)])  # in the channels that rotation leaves alone
    wq, wk = w["l0.mix.q"].astype(np.float64).copy(), w["l0.mix.k"].astype(np.float64).copy()
    wq[3 * D:4 * D] += 6.0 * np.outer(d, dual[:, 1])  # head 3 on key head 1
    wk[1 * D:2 * D] += 6.0 * np.outer(d, dual[:, 0])
    w["l0.mix.q"], w["l0.mix.k"] = pl.round_bf16(wq.astype(np.float32)), pl.round_bf16(wk.astype(np.float32))
    toks = rng.choice(ids[2:], n).astype(np.int32)
    keys = [7, 38, 45]
    queries = sorted({k + size + o for k in keys for o in (-1, 0, 1) if k + size + o not in keys and k + size + o > k})
    toks[keys] = ids[0]
    toks[queries] = ids[1]
    ref, att = _probe(cfg, w, toks, "attention")
    a = att[0][3]
    inside = [(k + size - 1, k) for k in keys if k + size - 1 in queries]
    assert all(a[i, k] > 0.9 for i, k in inside) and (inside or size == 1)
    assert all(a[k + size, k] == 0.0 for k in keys)
    for other in (size - 1, size + 1, 0):  # a window that is one token off shows (0: no window)
        if other == 0 and size == 1:
            continue
        cfg2 = json.loads(json.dumps(cfg))
        cfg2["layers"][0]["mixer"]["mask"] = {"size": other} if other else None
        assert tl.rel_err(po.forward(w, cfg2, toks)[queries], ref[queries]) > 1e-2, other
    for dtype, tol in (("float32", 3e-5), ("bfloat16", 4e-2)):
        m = make(cfg, w, dtype, page_tokens=16)
        assert tl.rel_err(run_whole(m, toks), ref) < tol
        assert tl.rel_err(run_cut(m, toks, sorted({keys[0] + size - 1, keys[0] + size, keys[1] + size, keys[1] + size + 2})), ref) < tol
        assert tl.rel_err(run_cut(m, toks, [size // 2 + 1, size + size // 2 + 2, 2 * size + 5]), ref) < tol
        assert tl.rel_err(run_cut(m, toks, range(keys[0] + size - 2 if size > 1 else 5, n)), ref) < tol  # decoded one by one over the edges
        m.close()


def test_every_constant_shows():
    """Rotation constants, scales, biases, head offsets, the value norm's epsilon, mix factors, layer factors and the router's correction
    each move the logits clearly when they are a little off."""
    cfg = pl.config([pl.attn_layer(size=64, scale=1.2, mlp=pl.dense()), pl.attn_layer(size=30, scale=1.2, mlp=pl.moe()), pl.latent_layer(scale=1.5, mlp=pl.moe(groups=(2, 1)))])
    w = pl.weights(cfg, seed=27)
    toks = pl.tokens(28, 150, cfg["vocab"])
    ref = po.forward(w, cfg, toks)
    changes = [lambda c: c["layers"][0]["mixer"]["rot"].update(base=800.0), lambda c: c["layers"][0]["mixer"]["rot"].update(dims=8),
               lambda c: c["layers"][2]["mixer"]["rot"].update(base=2000.0), lambda c: c["layers"][2]["mixer"].update(scale=1.4),
               lambda c: c["layers"][1]["mixer"].update(scale=1.1), lambda c: c["layers"][1]["mixer"].update(v_mix=False),
               lambda c: c["layers"][0]["mixer"].update(v_mix=False), lambda c: c["norm"].update(eps=1e-2),
               lambda c: c["layers"][1]["mlp"]["router"].update(groups={"count": 4, "keep": 1}), lambda c: c["layers"][2]["mlp"]["router"].pop("groups")]
    for i, change in enumerate(changes):
        cfg2 = json.loads(json.dumps(cfg))
        change(cfg2)
        assert tl.rel_err(po.forward(w, cfg2, toks), ref) > 1e-3, i
    for name in ("l0.mix.q.b", "l0.mix.k.b", "l0.mix.v.b", "l0.mix.o.b", "l0.mix.pb", "l1.mix.vmix", "l1.mlp.correction", "l2.mix.sink", "l0.ls1", "l1.ls2",
                 "l1.mlp.shared.sg"):
        w2 = dict(w)
        w2[name] = np.zeros_like(w[name])
        assert tl.rel_err(po.forward(w2, cfg, toks), ref) > 1e-3, name
    m = make(cfg, w)
    tl.assert_close(run_whole(m, toks), ref, "float32")
    tl.assert_close(run_cut(m, toks, [5, 60, 66, 130] + list(range(131, 150))), ref, "float32")
    m.close()


def test_small_values_meet_the_epsilon_of_their_norm():
    """Value heads whose mean square is of the size of the epsilon: it stands inside the root."""
    cfg = pl.config([pl.attn_layer(mlp=None), pl.attn_layer(heads=2)], eps=1e-3)
    w = pl.weights(cfg, seed=37)
    for n in ("l0.mix.v", "l0.mix.v.b"):
        w[n] = pl.round_bf16(0.03 * w[n])
    toks = pl.tokens(37, 60, cfg["vocab"])
    ref = po.forward(w, cfg, toks)
    m = make(cfg, w)
    tl.assert_close(run_whole(m, toks), ref, "float32")
    tl.assert_close(run_cut(m, toks, range(20, 60)), ref, "float32")
    m.close()


def test_pass_through_choices_and_dropped_groups():
    """Stacks whose routers choose only pass-through outputs, only experts, or a mix (asserted), with choice scores below zero in every
    group: prompts, ragged portions and decode steps."""
    for seed, corr in ((1, [-9, -9, -9, -9, 0, 0]), (2, [0, 0, 0, 0, -9, -9]), (3, [-1.0, -1.2, -1.1, -1.0, -1.1, -0.9])):
        cfg = pl.config([pl.latent_layer(mlp=pl.moe(experts=4, identity=2, groups=(3, 2), top=2)), pl.attn_layer(mlp=pl.moe(experts=4, identity=2, groups=(3, 1), top=2, shared=0))])
        w = pl.weights(cfg, seed=40 + seed, router_std=3.0)
        for p in ("l0.", "l1."):
            w[p + "mlp.correction"] = pl.round_bf16(np.array(corr, np.float32))
        toks = pl.tokens(43, 60, cfg["vocab"])
        po.PROBE = []
        try:
            ref = po.forward(w, cfg, toks)
            picks = [p[1] for p in po.PROBE if p[0] == "router"]
        finally:
            po.PROBE = None
        through = (picks[1] >= 4).mean()
        assert through == {1: 1.0, 2: 0.0}.get(seed, through) and (seed != 3 or 0.0 < through < 1.0)
        m = make(cfg, w)
        tl.assert_close(run_whole(m, toks), ref, "float32", seed)
        tl.assert_close(run_cut(m, toks, [3, 5, 30, 31] + list(range(40, 60))), ref, "float32", seed)
        m.close()


def test_first_tokens_and_single_token_sequences():
    cfg = full_cfg()
    w = pl.weights(cfg, seed=12)
    m = make(cfg, w)
    for n in (1, 2, 3, 6):
        toks = pl.tokens(50 + n, n, cfg["vocab"])
        ref = po.forward(w, cfg, toks)
        tl.assert_close(run_whole(m, toks), ref, "float32")
        tl.assert_close(run_cut(m, toks, range(1, n)), ref, "float32")
    m.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(dtype):
    cfg = full_cfg()
    w = pl.weights(cfg, seed=13)
    toks = pl.tokens(60, 200, cfg["vocab"])
    ref = po.forward(w, cfg, toks)
    m = make(cfg, w, dtype, page_tokens=8)
    got = run_cut(m, toks, range(8, 200))
    tl.assert_close(got, ref, dtype)
    m.close()


def test_decoding_with_split_rows_across_length_buckets():
    """Attention without a window: decode steps replay a graph per bucket of the longest sequence's length (512, 1024, ... tokens), and rows of
    more than 512 keys are shared between workgroups.  Two sequences decode in lock step while the longer one crosses 512 and 1024; a
    window of 700 positions beside it."""
    cfg = pl.config([pl.attn_layer(heads=4, kv_heads=2, dim=8, size=0), pl.attn_layer(heads=6, kv_heads=2, dim=6, size=700)], width=24, vocab=61)
    w = pl.weights(cfg, seed=31)
    a, b = pl.tokens(65, 1040, cfg["vocab"]), pl.tokens(66, 560, cfg["vocab"])
    ra, rb = po.forward(w, cfg, a), po.forward(w, cfg, b)
    m = make(cfg, w, max_tokens=2048)
    sa, sb = m.open(), m.open()
    m.step([(sa, a[:505], []), (sb, b[:25], [])])
    for lo, n in ((505, 15), (1015, 25)):  # 505 .. 519 and 1015 .. 1039 of the longer sequence
        if lo == 1015:
            m.step([(sa, a[520:1015], []), (sb, b[40:535], [])])
        rows = [m.step([(sa, a[lo + t:lo + t + 1], [0]), (sb, b[lo - 480 + t:lo - 479 + t], [0])]) for t in range(n)]
        tl.assert_close(np.stack([r[0] for r in rows]), ra[lo:lo + n], "float32", lo)
        tl.assert_close(np.stack([r[1] for r in rows]), rb[lo - 480:lo - 480 + n], "float32", lo)
    m.close()


def test_decode_steps_with_and_without_the_captured_graph():
    """A decode step replays the graph captured for its batch size; every replay, with eager prompt steps of other sequences between them,
    equals the same step launched kernel by kernel."""
    cfg = full_cfg()
    w = pl.weights(cfg, seed=17)
    a, b = pl.tokens(63, 40, cfg["vocab"]), pl.tokens(64, 25, cfg["vocab"])
    outs = []
    for use_graph in (True, False):
        m = make(cfg, w, use_graph=use_graph)
        sa, sb = m.open(), m.open()
        rows = [m.step([(sa, a[:10], [9])])]
        for t in range(10, 40):
            rows.append(m.step([(sa, a[t:t + 1], [0])]))
            if t % 7 == 0:  # eager work of another sequence between two replays
                lo = (t // 7 - 1) * 5
                rows.append(m.step([(sb, b[lo:lo + 5], [4])]))
        outs.append(np.concatenate(rows))
        m.close()
    assert np.array_equal(outs[0], outs[1])


def test_larger_odd_sizes_take_the_tiled_products():
    """Sizes that are not multiples of the kernels' tiles and vectors, enough rows for every tiled form, a width no vector load divides, rows
    beyond the register-held norms."""
    cfg = pl.config([pl.attn_layer(heads=2, kv_heads=1, dim=128, vdim=100, scale=0.09, size=150, rot_dims=100, mlp=pl.dense(ff=101)),
                     pl.latent_layer(heads=5, dim=20, vdim=30, rot_dim=10, kv_rank=60, scale=0.2, mlp=pl.moe(ff=51, shared=77)),
                     pl.attn_layer(heads=3, kv_heads=1, dim=64, vdim=100, scale=0.12, size=0, mlp=pl.moe(ff=65, experts=14, identity=2, groups=(4, 3), top=4, shared=101)),
                     pl.attn_layer(heads=1, kv_heads=1, dim=200, vdim=100, scale=0.07, size=40)], vocab=203, width=77)
    w = pl.weights(cfg, seed=14)
    toks = pl.tokens(61, 330, cfg["vocab"])
    ref = po.forward(w, cfg, toks)
    for dtype in ("float32", "bfloat16"):
        m = make(cfg, w, dtype)
        tl.assert_close(run_whole(m, toks), ref, dtype, dtype)
        tl.assert_close(run_cut(m, toks, [7, 140, 141, 215, 325]), ref, dtype, dtype)
        m.close()
    wide = pl.config([pl.attn_layer(mlp=pl.moe(ff=3, shared=2)), pl.latent_layer(mlp=pl.dense(ff=5))], width=4100, vocab=50)
    w = pl.weights(wide, seed=15)
    toks = pl.tokens(62, 12, 50)
    m = make(wide, w)
    tl.assert_close(run_cut(m, toks, [9, 10]), po.forward(w, wide, toks), "float32")
    m.close()


def test_greedy_and_sampled_generation():
    cfg = full_cfg()
    w = pl.weights(cfg, seed=15)
    prompts = [pl.tokens(70, 9, cfg["vocab"]), pl.tokens(71, 2, cfg["vocab"]), pl.tokens(72, 30, cfg["vocab"])]
    m = make(cfg, w, max_step_tokens=16)
    total = m.free_tokens()
    got = m.generate(prompts, 12)
    for p, g in zip(prompts, got):
        seq = po.Sequence(cfg)
        lg = po.forward(w, cfg, p, seq)
        for t in range(12):
            order = np.argsort(-lg[-1])
            if lg[-1][order[0]] - lg[-1][order[1]] < 1e-3 * np.abs(lg[-1]).max():
                break  # a near tie: fp32 and fp64 may differ from here on
            assert g[t] == order[0], (t, g, order[:3])
            lg = po.forward(w, cfg, [int(g[t])], seq)
    assert m.free_tokens() == total  # generate gave every slot and page back
    a = m.generate(prompts, 10, temp=2.0, seed=3)
    assert np.array_equal(a, m.generate(prompts, 10, temp=2.0, seed=3)) and not np.array_equal(a, m.generate(prompts, 10, temp=2.0, seed=4))
    assert np.array_equal(m.generate(prompts, 4, temp=1e-3, seed=1), got[:, :4])
    m.close()


def test_checkpoint_folder_through_registry_host_program_and_trace_replay(tmp_path):
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg = full_cfg()
    w = pl.weights(cfg, seed=16)
    path = str(tmp_path / "ckpt")
    os.makedirs(path)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    weights_io.write_safetensors(os.path.join(path, "model.safetensors"), w)
    prompts = [pl.tokens(80, 11, cfg["vocab"]), pl.tokens(81, 4, cfg["vocab"])]
    m = models.load_model(path, dtype="float32", max_tokens=256, max_seqs=4)
    assert isinstance(m, lm.LayeredLM) and m.config.architecture == "Pemuvik" and m.config.layers[1].identity == 2
    want = m.generate(prompts, 9)
    ref = po.forward(w, cfg, prompts[0])
    s = m.open()
    tl.assert_close(m.step([(s, prompts[0], list(range(11)))]), ref, "float32")
    m.close()
    exe = os.path.join(root, "zig_gpt2_amd", "bin", "zgpt2_main")
    arg = ";".join(",".join(str(int(t)) for t in p) for p in prompts)
    out = subprocess.run([exe, "lm", path, arg, "9", "--dtype", "float32"], capture_output=True, text=True, timeout=120)
    assert out.returncode == 0, out.stderr
    got = np.array([[int(t) for t in line.split()] for line in out.stdout.strip().splitlines()])
    assert np.array_equal(got, want)
    a, b = [int(t) for t in prompts[0]], [int(t) for t in prompts[1]]
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:6], "want": [5]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[6:9], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b, "want": [0, 3]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": a[9:10], "want": [0]}], "end": []},
             {"step": 4, "entries": [{"id": "a", "tokens": a[10:11], "want": [0]}], "end": ["a"]},
             {"step": 5, "entries": [{"id": "c", "tokens": a, "want": [10]}], "end": ["c"]}]
    outdir = tmp_path / "out"
    for dtype in ("float32", "bfloat16"):
        run = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", path, "--dtype", dtype, "--out", str(outdir),
                              "--max-tokens", "64"], input="\n".join(json.dumps(x) for x in steps) + "\n", capture_output=True, text=True, timeout=300)
        assert run.returncode == 0, run.stderr
        assert [l for l in run.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(6)]
        refb = po.forward(w, cfg, prompts[1])
        rd = lambda i: np.fromfile(str(outdir / f"{i}.f32"), dtype="<f4").reshape(-1, cfg["vocab"])  # noqa: E731
        assert not (outdir / "1.f32").exists()
        tol = 3e-5 if dtype == "float32" else 4e-2
        for i, want_rows in ((0, ref[5:6]), (2, refb[[0, 3]]), (3, ref[9:10]), (4, ref[10:11]), (5, ref[10:11])):
            assert tl.rel_err(rd(i), want_rows) < tol, (dtype, i)


def test_scheduler_serves_more_requests_than_slots():
    """Continuous batching: seven requests of unequal lengths on two slots — every request's tokens equal its generation alone, slots and
    pages go round."""
    cfg = full_cfg()
    w = pl.weights(cfg, seed=18)
    m = make(cfg, w, max_tokens=128, max_seqs=2, page_tokens=8)
    reqs = [(pl.tokens(90 + i, n, cfg["vocab"]), k) for i, (n, k) in enumerate([(30, 6), (3, 9), (17, 2), (1, 12), (41, 5), (8, 8), (2, 1)])]
    alone = [m.generate([p], k)[0] for p, k in reqs]
    total = m.free_tokens()
    sch = lm.Scheduler(m, portion=16)
    ids = [sch.submit(p, k) for p, k in reqs]
    out = sch.run()
    for rid, want in zip(ids, alone):
        assert np.array_equal(out[rid], want), (rid, out[rid], want)
    assert m.free_tokens() == total and sch._reserved == 0
    assert sch.steps < sum(-(-len(p) // 16) + k for p, k in reqs)  # requests shared steps
    m.close()


def test_errors_are_reported():
    def refused(layers, spec=None):
        c = lm.LMConfig.from_json(pl.config(layers))
        if spec:
            spec(c)
        with pytest.raises(Exception):
            lm.LayeredLM(c, dtype="float32", max_tokens=64, max_seqs=1)

    refused([pl.attn_layer(), pl.attn_layer(kv_heads=1)])  # values of another shape to mix in
    refused([pl.attn_layer(), pl.attn_layer(vdim=9)])
    refused([pl.attn_layer(rot_dims=5)])
    refused([pl.attn_layer(heads=3, kv_heads=2)])
    refused([pl.latent_layer(mlp=pl.moe(experts=6, identity=1, groups=(2, 1)))])  # seven outputs in two groups
    refused([pl.latent_layer(mlp=pl.moe(experts=6, identity=2, groups=(4, 1), top=3))])  # more chosen than the kept group holds
    refused([pl.latent_layer(mlp=pl.moe(experts=250, identity=8, groups=None))])
    refused([pl.latent_layer(mlp=pl.moe())], lambda c: setattr(c.layers[0], "router", "sigmoid_groups"))  # pass-through outputs of another rule
    refused([pl.latent_layer()], lambda c: setattr(c.layers[0], "sigmoid_weights", True))
    cfg = pl.config([pl.attn_layer(mlp=pl.dense()), pl.attn_layer()])
    w = pl.weights(cfg, seed=3)
    m = lm.LayeredLM(lm.LMConfig.from_json(cfg), dtype="float32", max_tokens=64, max_seqs=1)
    s = m.open()
    with pytest.raises(Exception):
        m.step([(s, [1, 2], [0])])  # no weights yet
    missing = w.pop("l1.mix.vmix")
    with pytest.raises(KeyError):
        m.load_weights(w)
    del w["l0.mix.vmix"]  # the first layer's is not read
    w["l1.mix.vmix"] = missing
    m.load_weights(w)
    m.close()


def _random_cfg(rng):
    """A stack with sizes drawn at random: odd and even widths, grouped heads, both mixers in any order, layers with and without a
    feed-forward, value mixing in some of the attention layers."""
    layers, shape = [], (int(rng.choice([1, 2, 3])), int(rng.integers(1, 40)))  # key heads and value channels of the layers that mix
    for i in range(int(rng.integers(1, 7))):
        mlp = None
        if rng.random() < 0.85:
            if rng.random() < 0.4:
                mlp = pl.dense(ff=int(rng.integers(1, 90)))
            else:
                n, per = int(rng.choice([1, 2, 3, 5])), int(rng.integers(1, 7))
                keep = int(rng.integers(1, n + 1))
                identity = int(rng.integers(0, n * per))
                mlp = pl.moe(ff=int(rng.integers(1, 50)), experts=n * per - identity, identity=identity, groups=(n, keep), top=int(rng.integers(1, keep * per + 1)),
                             shared=int(rng.integers(1, 60)) if rng.random() < 0.7 else 0)
        if rng.random() < 0.35:
            layers.append(pl.latent_layer(heads=int(rng.integers(1, 6)), dim=int(rng.integers(1, 30)), vdim=int(rng.integers(1, 30)), scale=float(rng.choice([0.1, 0.5, 1.5])),
                                          kv_rank=int(rng.integers(1, 90)), rot_dim=2 * int(rng.integers(1, 9)), base=float(rng.choice([50.0, 10000.0])), mlp=mlp))
        else:
            mixes = rng.random() < 0.7
            kv, vdim = shape if mixes else (int(rng.choice([1, 2, 3])), int(rng.integers(1, 90)))
            dim = int(rng.integers(2, 90))
            layers.append(pl.attn_layer(heads=kv * int(rng.choice([1, 2, 4, 5])), kv_heads=kv, dim=dim, vdim=vdim, scale=float(rng.choice([0.05, 0.2, 0.6])),
                                        size=int(rng.choice([0, 1, 2, 7, 16, 33, 100, 1000])), rot_dims=2 * int(rng.integers(0, dim // 2 + 1)),
                                        base=float(rng.choice([100.0, 10000.0])), v_mix=mixes, mlp=mlp))
    return pl.config(layers, vocab=int(rng.integers(2, 300)), width=int(rng.integers(3, 90)), eps=float(rng.choice([1e-6, 1e-5, 1e-3])))


@pytest.mark.parametrize("seed", range(16))
def test_sizes_drawn_at_random(seed):
    rng = np.random.default_rng(9100 + seed)
    cfg = _random_cfg(rng)
    w = pl.weights(cfg, seed=seed)
    n = int(rng.integers(20, 300))
    toks = pl.tokens(seed, n, cfg["vocab"])
    ref = po.forward(w, cfg, toks)
    m = make(cfg, w, page_tokens=int(rng.choice([4, 16, 64])))
    tl.assert_close(run_whole(m, toks), ref, "float32", cfg)
    cuts = sorted(set(int(c) for c in rng.integers(1, n, 6))) + list(range(max(1, n - 12), n))
    tl.assert_close(run_cut(m, toks, sorted(set(cuts))), ref, "float32", (cfg, cuts))
    m.close()
