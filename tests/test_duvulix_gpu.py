"""The Duvulix design on the layered-model tier (zig_gpt2_amd/lm.py) against the float64 oracle of tests/duvulix_oracle.py: every
mechanism alone, whole prompts against portions and token-by-token decoding, ragged batches, slots and pages that go round, heavy
keys hundreds of tokens back and on both sides of a chunk's edge, latents that several layers read, states that forget slowly and
at once across the chunks of the recurrence, other sizes, and generation through the library's entry points, the scheduler, the
host program and the trace replay."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import duvulix_oracle as do
import duvulix_testlib as dl
import lm_testlib as tl
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
    "mamba": [dl.mamba_layer()],
    "mamba_one_head": [dl.mamba_layer(heads=1, vdim=3, state=1, groups=1, conv=4)],
    "mamba_own_groups": [dl.mamba_layer(heads=5, vdim=4, state=7, groups=5, conv=2, norm_groups=4)],  # every head its own B and C; rows no vector load divides
    "mamba_no_window": [dl.mamba_layer(heads=6, vdim=8, state=40, groups=2, conv=1, norm_groups=3)],  # one tap: nothing carried by the convolution
    "mamba_long_taps": [dl.mamba_layer(heads=3, vdim=34, state=33, groups=1, conv=7, norm_groups=2)],  # beyond the taps held in registers, ragged tiles
    "mamba_wide_values": [dl.mamba_layer(heads=2, vdim=130, state=20, groups=1, norm_groups=1)],  # more column tiles than a workgroup has waves
    "latent": [dl.latent_layer()],
    "latent_one_head": [dl.latent_layer(heads=1, dim=3, vdim=5, rot_dim=2, kv_rank=9, scale=0.9)],
    "latent_shared": [dl.latent_layer(), dl.latent_layer(heads=2, dim=4, vdim=3, kv_from=0), dl.latent_layer(heads=5, dim=7, vdim=2, scale=0.6, kv_from=0)],
    "latent_shared_apart": [dl.latent_layer(), dl.latent_layer(kv_rank=11, rot_dim=4), dl.latent_layer(kv_from=0), dl.latent_layer(kv_rank=11, rot_dim=4, kv_from=1)],
    "attention": [dl.attn_layer()],  # grouped keys, chunks, blended frequencies
    "attention_own_keys": [dl.attn_layer(heads=3, kv_heads=3, dim=8, vdim=8, size=5, scaling=None)],
    "attention_partial_rotation": [dl.attn_layer(heads=5, kv_heads=1, dim=7, vdim=3, rot_dims=4, size=16)],  # odd channels, the last three pass
    "attention_chunks_of_one": [dl.attn_layer(size=1)],  # every token sees itself
    "attention_whole_context": [dl.attn_layer(size=0, rot_dims=0)],  # no chunks, no rotation
    "attention_wide_heads": [dl.attn_layer(heads=2, kv_heads=1, dim=150, vdim=66, scale=0.05, size=20)],  # beyond the tiled scores
    "ff": [dl.mamba_layer(mlp=dl.dense())],
    "ff_narrow": [dl.attn_layer(mlp=dl.dense(ff=1)), dl.latent_layer(mlp=dl.dense(ff=7))],
    "ff_long_rows": [dl.attn_layer(mlp=dl.dense(ff=1700))],  # second products that split their rows over waves
    "ff_longer_than_registers": [dl.attn_layer(mlp=dl.dense(ff=4300))],
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(SINGLE))
def test_each_mechanism_alone(name, dtype):
    cfg = dl.config(SINGLE[name], width=50 if "one_head" in name else 40)
    w = dl.weights(cfg, seed=sum(map(ord, name)))
    toks = dl.tokens(1, 83 if "one_head" in name or "long_taps" in name else 37, cfg["vocab"])
    ref_tr = []
    ref = do.forward(w, cfg, toks, trace=ref_tr)
    m = make(cfg, w, dtype)
    got, tr = run_whole(m, toks, trace=True)
    tl.assert_close(tr, np.stack(ref_tr), dtype, "residual stream")
    tl.assert_close(got, ref, dtype, "logits")
    # the same prompt token by token: the decode kernels, state carried by the slot
    step = run_cut(m, toks, range(1, len(toks)))
    tl.assert_close(step, ref, dtype, "decoded")
    m.close()


def full_cfg(**kw):
    return dl.config([dl.mamba_layer(mlp=dl.dense()), dl.latent_layer(mlp=dl.dense(ff=50)), dl.latent_layer(heads=2, dim=5, vdim=9, kv_from=1, mlp=dl.dense()),
                      dl.attn_layer(mlp=None), dl.mamba_layer(heads=6, vdim=6, state=9, groups=3, conv=4, norm_groups=2, mlp=dl.dense(ff=13)),
                      dl.attn_layer(heads=6, kv_heads=3, dim=4, vdim=5, scale=0.5, size=14, rot_dims=2, mlp=dl.dense()),
                      dl.latent_layer(heads=1, kv_rank=7, rot_dim=4, mlp=None), dl.latent_layer(heads=4, kv_from=1, mlp=dl.dense())], **kw)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_portions_of_several_sizes(dtype):
    cfg = full_cfg()
    w = dl.weights(cfg, seed=5)
    toks = dl.tokens(2, 90, cfg["vocab"])
    ref = do.forward(w, cfg, toks)
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
    w = dl.weights(cfg, seed=7)
    lens = [41, 3, 17, 1]
    prompts = [dl.tokens(10 + i, n, cfg["vocab"]) for i, n in enumerate(lens)]
    refs = [do.forward(w, cfg, p) for p in prompts]
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
    more = [dl.tokens(20 + i, 6, cfg["vocab"]) for i in range(3)]
    alone = [do.forward(w, cfg, np.concatenate([prompts[i], more[i]]))[len(prompts[i]):] for i in range(3)]
    rows = [m.step([(seqs[i], [more[i][t]], [0]) for i in range(3)]) for t in range(6)]
    for i in range(3):
        tl.assert_close(np.stack([r[i] for r in rows]), alone[i], dtype, i)
    m.close()


def test_decode_batches_of_every_size():
    """One to eight sequences in lock step, every batch size on its own captured graph (one and two rows apply the activation where the
    product reads it, more rows in a launch), each row against its sequence alone."""
    cfg = full_cfg()
    w = dl.weights(cfg, seed=9)
    m = make(cfg, w, max_seqs=8, page_tokens=8)
    seqs = [dl.tokens(100 + i, 5 + 3 * i + 9, cfg["vocab"]) for i in range(8)]
    refs = [do.forward(w, cfg, t) for t in seqs]
    slots = [m.open() for _ in seqs]
    at = [5 + 3 * i for i in range(8)]
    m.step([(s, t[:k], []) for s, t, k in zip(slots, seqs, at)])
    for n in (1, 2, 3, 4, 5, 6, 7, 8):
        got = m.step([(slots[i], [seqs[i][at[i]]], [0]) for i in range(n)])
        for i in range(n):
            tl.assert_close(got[i], refs[i][at[i]], "float32", (n, i))
            at[i] += 1
    m.close()


def test_slots_and_pages_are_reused():
    """Two slots and a cache of 96 tokens in pages of 4.  A closed sequence gives its pages and its slot back; the next one starts from
    an empty state and an empty convolution window, on pages that held other keys and latents."""
    cfg = full_cfg()
    w = dl.weights(cfg, seed=8)
    m = make(cfg, w, max_tokens=96, max_seqs=2, page_tokens=4)
    total = m.free_tokens()
    a, b, c = (dl.tokens(30 + i, n, cfg["vocab"]) for i, n in enumerate((50, 38, 44)))
    ra, rb, rc = (do.forward(w, cfg, t) for t in (a, b, c))
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


def test_chunked_sequences_outgrow_the_cache():
    """A stack that looks back one chunk at most returns the pages behind it while the sequence runs: 300 tokens through a cache of 64, in
    portions and decoded, two sequences taking each other's pages."""
    cfg = dl.config([dl.attn_layer(size=12, mlp=dl.dense()), dl.mamba_layer(), dl.attn_layer(heads=2, kv_heads=1, size=20)])
    w = dl.weights(cfg, seed=33)
    a, b = dl.tokens(34, 300, cfg["vocab"]), dl.tokens(35, 300, cfg["vocab"])
    ra, rb = do.forward(w, cfg, a), do.forward(w, cfg, b)
    m = make(cfg, w, max_tokens=64, max_seqs=2, page_tokens=4)
    total = m.free_tokens()
    sa, sb = m.open(), m.open()
    lo = 0
    for n in [7, 2, 12, 3, 1, 1, 9, 11, 2, 5] * 5 + [12] * 2 + [1] * 11:
        got = m.step([(sa, a[lo:lo + n], list(range(n))), (sb, b[lo:lo + n], list(range(n)))])
        tl.assert_close(got[:n], ra[lo:lo + n], "float32", lo)
        tl.assert_close(got[n:], rb[lo:lo + n], "float32", lo)
        lo += n
    assert lo == 300 and total - m.free_tokens() <= 2 * 28
    m.close_seq(sa)
    m.close_seq(sb)
    assert m.free_tokens() == total
    m.close()


def test_general_attention_kernel(monkeypatch):
    """The one-workgroup-per-row form of the chunked attention (what a step takes when the split form's workspace would not fit), on
    prompts, portions and decoded tokens over several key tiles."""
    monkeypatch.setenv("ZGPT2_LM_WINDOW_GENERAL", "1")
    cfg = dl.config([dl.attn_layer(size=90), dl.attn_layer(heads=2, kv_heads=1, dim=70, vdim=40, scale=0.08, size=33), dl.attn_layer(size=0)])
    w = dl.weights(cfg, seed=21)
    toks = dl.tokens(22, 200, cfg["vocab"])
    ref = do.forward(w, cfg, toks)
    for dtype in ("float32", "bfloat16"):
        m = make(cfg, w, dtype)
        tl.assert_close(run_whole(m, toks), ref, dtype)
        tl.assert_close(run_cut(m, toks, [3, 64, 65, 130] + list(range(180, 200))), ref, dtype)
        m.close()


@pytest.mark.parametrize("hook", ["ZGPT2_LM_WINDOW_NO_TILES", "ZGPT2_LM_WINDOW_TILES", "ZGPT2_LM_SSD_NO_CHUNKS"])
def test_both_forms_of_a_kernel_on_all_steps(monkeypatch, hook):
    """Prompt portions take scores from matrix-core tiles and states from chunks of tokens, steps of few rows from the per-key kernel and
    the token-by-token scan; the hooks send every step through one of them (ragged row blocks, two entries)."""
    monkeypatch.setenv(hook, "1")
    cfg = dl.config([dl.attn_layer(heads=6, kv_heads=2, dim=18, size=40), dl.attn_layer(heads=1, kv_heads=1, dim=5, vdim=1, rot_dims=4, size=33),
                     dl.mamba_layer(heads=6, vdim=33, state=18, groups=2), dl.attn_layer(heads=18, kv_heads=6, dim=4, scale=0.7, size=70)])
    w = dl.weights(cfg, seed=23)
    a, b = dl.tokens(24, 150, cfg["vocab"]), dl.tokens(25, 47, cfg["vocab"])
    ra, rb = do.forward(w, cfg, a), do.forward(w, cfg, b)
    m = make(cfg, w)
    tl.assert_close(run_whole(m, a), ra, "float32")
    tl.assert_close(run_cut(m, a, [3, 35, 36, 100] + list(range(140, 150))), ra, "float32")
    sa, sb = m.open(), m.open()
    got = m.step([(sa, a[:70], list(range(70))), (sb, b, list(range(47)))])
    tl.assert_close(got[:70], ra[:70], "float32")
    tl.assert_close(got[70:], rb, "float32")
    m.close()


def _probe(cfg, w, toks, kind):
    do.PROBE = []
    try:
        ref = do.forward(w, cfg, toks)
        att = [p[1] for p in do.PROBE if p[0] == kind]
    finally:
        do.PROBE = None
    return ref, att


def _input_duals(cfg, w, ids):
    """In the first layer the mixer's input depends on the token alone.  Column t of the result has a product of one with the input of
    token ids[t] and of zero with every other listed token's."""
    return np.linalg.pinv(do.offset_norm(w["l0.norm1"], w["embed"].astype(np.float64)[ids], cfg["norm"]["eps"]))


@pytest.mark.parametrize("shared", [False, True])
def test_far_latents_among_hundreds(shared):
    """One key is made to stand out: the latent of one token id gets a large component that no other token of the prompt has, one head's key
    projection reads it and that head's query of another token id asks for it.  It sits at position 5, its queries hundreds of tokens
    later — across pages, key tiles and the shares of a split row; once in the layer's own latents, once in a layer that reads another's."""
    n, W, KR = 420, 32, 16
    layers = [dl.latent_layer(heads=3, dim=12, vdim=6, rot_dim=6, kv_rank=KR, scale=0.5)]
    if shared:
        layers.append(dl.latent_layer(heads=3, dim=12, vdim=6, rot_dim=6, kv_rank=KR, scale=0.5, kv_from=0))
    cfg = dl.config(layers, width=W)
    w = dl.weights(cfg, seed=19)
    if shared:  # the first layer leaves the stream as it is, so the second one's input depends on the token alone too
        w["l0.mix.o"] = np.zeros_like(w["l0.mix.o"])
        w["l1.norm1"] = w["l0.norm1"].copy()
    p = "l1.mix." if shared else "l0.mix."
    rng = np.random.default_rng(19)
    ids = rng.permutation(cfg["vocab"])[:22]
    dual = _input_duals(cfg, w, ids)
    toks = rng.choice(ids[2:], n).astype(np.int32)
    queries = (230, 300, 301, 388, 419)
    toks[5], toks[list(queries)] = ids[0], ids[1]
    lat, d = rng.normal(0.0, 1.0, KR), rng.normal(0.0, 1.0, 12)
    dkv, uk, q = (w[k].astype(np.float64).copy() for k in ("l0.mix.dkv", p + "uk", p + "q"))
    dkv[:KR] += 30.0 * np.outer(lat, dual[:, 0])
    uk[12:24] += np.outer(d, lat) * 0.5  # head 1
    q[18:30] += 8.0 * np.outer(d, dual[:, 1])
    w["l0.mix.dkv"], w[p + "uk"], w[p + "q"] = (dl.round_bf16(a.astype(np.float32)) for a in (dkv, uk, q))
    ref, att = _probe(cfg, w, toks, "latent_attention")
    assert all(att[-1][1, i, 5] > 0.8 for i in queries), [att[-1][1, i, 5] for i in queries]
    gone = toks.copy()
    gone[5] = toks[6]
    assert tl.rel_err(do.forward(w, cfg, gone)[list(queries)], ref[list(queries)]) > 1e-2
    for dtype, tol in (("float32", 2e-4), ("bfloat16", 4e-2)):
        m = make(cfg, w, dtype, page_tokens=16)
        for got in (run_whole(m, toks), run_cut(m, toks, [4, 5, 6, 100, 229, 230, 231, 333] + list(range(380, n)))):
            assert tl.rel_err(got[list(queries)], ref[list(queries)]) < tol
            if dtype == "bfloat16":  # a sharp softmax of rounded operands: the module's statement about bfloat16 rows
                tl.assert_close(got, ref, dtype)
            else:
                assert tl.rel_err(got, ref) < tol
        m.close()


@pytest.mark.parametrize("size", [31, 32, 64, 100])
def test_heavy_keys_inside_and_outside_a_chunk(size):
    """One token id's key stands out for another's queries.  It sits in the last and in the first place of a chunk; queries sit in the
    same chunk (just inside its far edge too) and just behind the edge, where the key must weigh nothing."""
    n, W, D = 3 * size + 8, 32, 16
    cfg = dl.config([dl.attn_layer(heads=4, kv_heads=2, dim=D, vdim=10, scale=0.4, size=size, rot_dims=4)], width=W)
    w = dl.weights(cfg, seed=size)
    rng = np.random.default_rng(size)
    ids = rng.permutation(cfg["vocab"])[:22]
    dual = _input_duals(cfg, w, ids)
    d = np.concatenate([np.zeros(4), rng.normal(0.0, 1.0, D - 4)])  # in the channels that rotation leaves alone
    wq, wk = w["l0.mix.q"].astype(np.float64).copy(), w["l0.mix.k"].astype(np.float64).copy()
    wq[3 * D:4 * D] += 6.0 * np.outer(d, dual[:, 1])  # head 3 on key head 1
    wk[1 * D:2 * D] += 6.0 * np.outer(d, dual[:, 0])
    w["l0.mix.q"], w["l0.mix.k"] = dl.round_bf16(wq.astype(np.float32)), dl.round_bf16(wk.astype(np.float32))
    toks = rng.choice(ids[2:], n).astype(np.int32)
    first, last = size, 2 * size - 1  # the second chunk
    toks[[first, last - 1]] = ids[0]
    queries = [first + 1, last, last + 1, last + 2, 3 * size - 1, 3 * size]
    toks[queries] = ids[1]
    ref, att = _probe(cfg, w, toks, "attention")
    a = att[0][3]
    assert a[first + 1, first] > 0.8 and a[last, last - 1] + a[last, first] > 0.8
    assert all(a[i, first] == 0.0 and a[i, last - 1] == 0.0 for i in queries[2:])
    for other in (size - 1, size + 1, 2 * size, 0):  # a chunk that is one token off shows
        cfg2 = json.loads(json.dumps(cfg))
        cfg2["layers"][0]["mixer"]["mask"] = {"size": other} if other else None
        assert tl.rel_err(do.forward(w, cfg2, toks)[queries], ref[queries]) > 1e-2, other
    for dtype, tol in (("float32", 2e-4), ("bfloat16", 4e-2)):
        m = make(cfg, w, dtype, page_tokens=16)
        assert tl.rel_err(run_whole(m, toks), ref) < tol
        assert tl.rel_err(run_cut(m, toks, [first - 1, first, first + 2, last, last + 1, last + 3]), ref) < tol  # portions around the edges
        assert tl.rel_err(run_cut(m, toks, [size // 2, size + size // 2, 2 * size + 5]), ref) < tol  # cuts in the middle of chunks
        assert tl.rel_err(run_cut(m, toks, range(first - 3, n)), ref) < tol  # decoded one by one over both edges
        m.close()


def test_rotation_constants_show():
    """Each constant of the rotation moves the logits clearly when it is a little off, and so do the gate and the shared latents."""
    cfg = dl.config([dl.attn_layer(size=64, dim=12, scale=1.5), dl.latent_layer(scale=1.5), dl.latent_layer(scale=1.5, kv_from=1)])
    w = dl.weights(cfg, seed=27)
    toks = dl.tokens(28, 150, cfg["vocab"])
    ref = do.forward(w, cfg, toks)
    changes = [lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=5.0), lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(original=48),
               lambda c: c["layers"][0]["mixer"]["rot"].update(scaling=None), lambda c: c["layers"][0]["mixer"]["rot"].update(dims=10),
               lambda c: c["layers"][1]["mixer"]["rot"].update(base=4000.0), lambda c: c["layers"][2]["mixer"]["rot"].update(base=4000.0),
               lambda c: c["layers"][2]["mixer"].update(scale=1.4)]
    for i, change in enumerate(changes):
        cfg2 = json.loads(json.dumps(cfg))
        change(cfg2)
        assert tl.rel_err(do.forward(w, cfg2, toks), ref) > 3e-3, i
    for name in ("l1.mix.g", "l2.mix.g"):
        w2 = dict(w)
        w2[name] = np.zeros_like(w[name])
        assert tl.rel_err(do.forward(w2, cfg, toks), ref) > 1e-2, name
    m = make(cfg, w)
    tl.assert_close(run_whole(m, toks), ref, "float32")
    tl.assert_close(run_cut(m, toks, [5, 60, 66, 130] + list(range(131, 150))), ref, "float32")
    m.close()


def test_state_remembers_far_tokens_across_chunks():
    """Decays close to one: the state forgets slowly, so the first tokens still weigh in hundreds of tokens later — a state or a convolution
    window that is lost, reset or carried wrongly between portions, chunks of the long-step form or decode steps shows.  Long steps
    run chunks of 32 tokens side by side; cuts sit at, before and behind their edges."""
    cfg = dl.config([dl.mamba_layer(heads=4, vdim=16, state=20, groups=2, conv=4, norm_groups=2)], width=32)
    w = dl.weights(cfg, seed=11, rate=(0.002, 0.02), dt_bias=(-1.0, 0.5))
    n = 600
    toks = dl.tokens(41, n, cfg["vocab"])
    other = toks.copy()
    other[:40] = (other[:40] + 1) % cfg["vocab"]
    ref, ref_other = do.forward(w, cfg, toks), do.forward(w, cfg, other)
    assert tl.rel_err(ref_other[-1], ref[-1]) > 1e-3, "the construction does not carry the first tokens to the end"
    m = make(cfg, w, max_tokens=1024)
    tl.assert_close(run_whole(m, toks), ref, "float32")
    tl.assert_close(run_cut(m, toks, [2, 4, 31, 32, 33, 63, 64, 65, 127, 129, 385, 386]), ref, "float32")
    tl.assert_close(run_cut(m, toks, [300] + list(range(540, n))), ref, "float32")
    m.close()


def test_tokens_that_forget_everything_do_not_blur_the_decays_behind_them():
    """Step sizes that reach the hundreds (logarithms of the decay in the thousands) between tokens whose decays are close to one: what
    follows such a token must still be weighed by its own small logarithms."""
    cfg = dl.config([dl.mamba_layer(heads=2, vdim=16, state=20, groups=1, conv=2)], width=32)
    w = dl.weights(cfg, seed=12, rate=(6.0, 20.0), dt_bias=(-5.0, 0.3))
    ids = np.random.default_rng(12).permutation(cfg["vocab"])[:22]
    dual = _input_duals(cfg, w, ids)
    win = w["l0.mix.in"].astype(np.float64).copy()
    win[-2:] = 0.3 * win[-2:] + 300.0 * dual[:, 0][None, :]
    w["l0.mix.in"] = dl.round_bf16(win.astype(np.float32))
    toks = np.random.default_rng(13).choice(ids[1:], 200).astype(np.int32)
    toks[[3, 31, 32, 50, 63, 90, 130, 170]] = ids[0]
    ref = do.forward(w, cfg, toks)
    u = do.offset_norm(w["l0.norm1"], w["embed"].astype(np.float64)[toks], cfg["norm"]["eps"])
    dt = do.softplus((u @ win.T)[:, -2:] + w["l0.mix.dt_bias"].astype(np.float64))
    assert dt[50].min() > 200 and np.median(dt) < 0.1
    m = make(cfg, w)
    tl.assert_close(run_whole(m, toks), ref, "float32")
    tl.assert_close(run_cut(m, toks, [31, 32, 33, 64, 120] + list(range(165, 200))), ref, "float32")
    m.close()


def test_first_tokens_and_single_token_sequences():
    cfg = full_cfg()
    w = dl.weights(cfg, seed=12)
    m = make(cfg, w)
    for n in (1, 2, 3, 6):
        toks = dl.tokens(50 + n, n, cfg["vocab"])
        ref = do.forward(w, cfg, toks)
        tl.assert_close(run_whole(m, toks), ref, "float32")
        tl.assert_close(run_cut(m, toks, range(1, n)), ref, "float32")
    m.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(dtype):
    cfg = full_cfg()
    w = dl.weights(cfg, seed=13)
    toks = dl.tokens(60, 200, cfg["vocab"])
    ref = do.forward(w, cfg, toks)
    m = make(cfg, w, dtype, page_tokens=8)
    got = run_cut(m, toks, range(8, 200))
    tl.assert_close(got, ref, dtype)
    m.close()


def test_decoding_across_length_buckets():
    """Whole-context rotary attention: decode steps replay a graph per bucket of the longest sequence's length (512, 1024, ... tokens).
    Two sequences decode in lock step while the longer one crosses 512 and 1024; a chunk of 700 positions beside it."""
    cfg = dl.config([dl.attn_layer(heads=4, kv_heads=2, dim=8, size=0), dl.mamba_layer(heads=1, vdim=8, groups=1), dl.attn_layer(heads=2, kv_heads=1, dim=6, size=700)],
                    width=24, vocab=61)
    w = dl.weights(cfg, seed=31)
    a, b = dl.tokens(65, 1040, cfg["vocab"]), dl.tokens(66, 560, cfg["vocab"])
    ra, rb = do.forward(w, cfg, a), do.forward(w, cfg, b)
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
    w = dl.weights(cfg, seed=17)
    a, b = dl.tokens(63, 40, cfg["vocab"]), dl.tokens(64, 25, cfg["vocab"])
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
    """Sizes that are not multiples of the kernels' tiles and vectors, enough rows for every tiled form, a state of more than 128 rows, a
    latent beyond the tiled prompt attention, a width no vector load divides, rows beyond the register-held norms."""
    cfg = dl.config([dl.mamba_layer(heads=6, vdim=40, state=130, groups=3, conv=4, norm_groups=5, mlp=dl.dense(ff=101)),
                     dl.latent_layer(heads=5, dim=20, vdim=30, rot_dim=10, kv_rank=60, scale=0.2, mlp=dl.dense(ff=300)),
                     dl.latent_layer(heads=2, dim=20, vdim=30, rot_dim=20, kv_rank=340, scale=0.2),
                     dl.attn_layer(heads=2, kv_heads=1, dim=128, vdim=100, scale=0.09, size=150), dl.mamba_layer(heads=3, vdim=70, state=256, groups=1, conv=4)],
                    vocab=203, width=77)
    w = dl.weights(cfg, seed=14)
    toks = dl.tokens(61, 330, cfg["vocab"])
    ref = do.forward(w, cfg, toks)
    for dtype in ("float32", "bfloat16"):
        m = make(cfg, w, dtype)
        tl.assert_close(run_whole(m, toks), ref, dtype, dtype)
        tl.assert_close(run_cut(m, toks, [7, 140, 141, 215, 325]), ref, dtype, dtype)
        m.close()
    wide = dl.config([dl.mamba_layer(heads=2, vdim=2100, state=3, groups=1, norm_groups=1), dl.attn_layer()], width=4100, vocab=50)
    w = dl.weights(wide, seed=15)
    toks = dl.tokens(62, 12, 50)
    m = make(wide, w)
    tl.assert_close(run_cut(m, toks, [9, 10]), do.forward(w, wide, toks), "float32")
    m.close()


def test_greedy_and_sampled_generation():
    cfg = full_cfg()
    w = dl.weights(cfg, seed=15)
    prompts = [dl.tokens(70, 9, cfg["vocab"]), dl.tokens(71, 2, cfg["vocab"]), dl.tokens(72, 30, cfg["vocab"])]
    m = make(cfg, w, max_step_tokens=16)
    total = m.free_tokens()
    got = m.generate(prompts, 12)
    for p, g in zip(prompts, got):
        seq = do.Sequence(cfg)
        lg = do.forward(w, cfg, p, seq)
        for t in range(12):
            order = np.argsort(-lg[-1])
            if lg[-1][order[0]] - lg[-1][order[1]] < 1e-3 * np.abs(lg[-1]).max():
                break  # a near tie: fp32 and fp64 may differ from here on
            assert g[t] == order[0], (t, g, order[:3])
            lg = do.forward(w, cfg, [int(g[t])], seq)
    assert m.free_tokens() == total  # generate gave every slot and page back
    a = m.generate(prompts, 10, temp=2.0, seed=3)
    assert np.array_equal(a, m.generate(prompts, 10, temp=2.0, seed=3)) and not np.array_equal(a, m.generate(prompts, 10, temp=2.0, seed=4))
    assert np.array_equal(m.generate(prompts, 4, temp=1e-3, seed=1), got[:, :4])
    m.close()


def test_checkpoint_folder_through_registry_host_program_and_trace_replay(tmp_path):
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg = full_cfg()
    w = dl.weights(cfg, seed=16)
    path = str(tmp_path / "ckpt")
    os.makedirs(path)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    weights_io.write_safetensors(os.path.join(path, "model.safetensors"), w)
    prompts = [dl.tokens(80, 11, cfg["vocab"]), dl.tokens(81, 4, cfg["vocab"])]
    m = models.load_model(path, dtype="float32", max_tokens=256, max_seqs=4)
    assert isinstance(m, lm.LayeredLM) and m.config.architecture == "Duvulix" and m.config.layers[2].kv_from == 1
    want = m.generate(prompts, 9)
    ref = do.forward(w, cfg, prompts[0])
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
        refb = do.forward(w, cfg, prompts[1])
        rd = lambda i: np.fromfile(str(outdir / f"{i}.f32"), dtype="<f4").reshape(-1, cfg["vocab"])  # noqa: E731
        assert not (outdir / "1.f32").exists()
        tol = 3e-5 if dtype == "float32" else 4e-2
        for i, want_rows in ((0, ref[5:6]), (2, refb[[0, 3]]), (3, ref[9:10]), (4, ref[10:11]), (5, ref[10:11])):
            assert tl.rel_err(rd(i), want_rows) < tol, (dtype, i)


def test_scheduler_serves_more_requests_than_slots():
    """Continuous batching: seven requests of unequal lengths on two slots — every request's tokens equal its generation alone, slots and
    pages go round."""
    cfg = full_cfg()
    w = dl.weights(cfg, seed=18)
    m = make(cfg, w, max_tokens=128, max_seqs=2, page_tokens=8)
    reqs = [(dl.tokens(90 + i, n, cfg["vocab"]), k) for i, (n, k) in enumerate([(30, 6), (3, 9), (17, 2), (1, 12), (41, 5), (8, 8), (2, 1)])]
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
    def refused(layers):
        with pytest.raises(Exception):
            lm.LayeredLM(lm.LMConfig.from_json(dl.config(layers)), dtype="float32", max_tokens=64, max_seqs=1)

    refused([dl.latent_layer(kv_from=1), dl.latent_layer()])  # latents that are not there yet
    refused([dl.mamba_layer(), dl.latent_layer(kv_from=0)])  # a layer without latents
    refused([dl.latent_layer(), dl.latent_layer(kv_rank=11, kv_from=0)])  # latents of another size
    refused([dl.latent_layer(), dl.latent_layer(kv_from=0), dl.latent_layer(kv_from=1)])  # a layer that has none of its own
    refused([dl.mamba_layer(state=300)])
    refused([dl.mamba_layer(heads=3, groups=2)])
    refused([dl.mamba_layer(heads=3, vdim=5, groups=1, norm_groups=2)])
    refused([dl.attn_layer(rot_dims=5)])
    cfg = dl.config([dl.mamba_layer(mlp=dl.dense())])
    w = dl.weights(cfg, seed=3)
    m = lm.LayeredLM(lm.LMConfig.from_json(cfg), dtype="float32", max_tokens=64, max_seqs=1)
    s = m.open()
    with pytest.raises(Exception):
        m.step([(s, [1, 2], [0])])  # no weights yet
    del w["l0.mlp.act"]
    with pytest.raises(KeyError):
        m.load_weights(w)
    m.close()


def _random_cfg(rng):
    """A stack with sizes drawn at random: odd and even widths, grouped heads, every kind of layer in any order, layers with and without a
    feed-forward, latent layers that read an earlier one's latents."""
    layers = []
    for i in range(int(rng.integers(1, 7))):
        mlp = dl.dense(ff=int(rng.integers(1, 90))) if rng.random() < 0.75 else None
        kind = rng.choice(["mamba", "latent", "attention"])
        if kind == "mamba":
            g, per = int(rng.choice([1, 2, 3])), int(rng.choice([1, 2, 3, 5]))
            vdim = int(rng.integers(1, 40))
            inner = g * per * vdim
            layers.append(dl.mamba_layer(heads=g * per, vdim=vdim, state=int(rng.integers(1, 70)), groups=g, conv=int(rng.integers(1, 7)),
                                         norm_groups=int(rng.choice([d for d in range(1, inner + 1) if inner % d == 0][:4])), mlp=mlp))
        elif kind == "latent":
            owners = [j for j, e in enumerate(layers) if e["type"] == "latent_attention" and "kv_from" not in e["mixer"]]
            kw = dict(heads=int(rng.integers(1, 6)), dim=int(rng.integers(1, 30)), vdim=int(rng.integers(1, 30)), scale=float(rng.choice([0.1, 0.5, 1.5])), mlp=mlp)
            if owners and rng.random() < 0.5:
                j = int(rng.choice(owners))
                m = layers[j]["mixer"]
                layers.append(dl.latent_layer(kv_from=j, kv_rank=m["kv_rank"], rot_dim=m["rot_dim"], base=m["rot"]["base"], **kw))
            else:
                layers.append(dl.latent_layer(kv_rank=int(rng.integers(1, 90)), rot_dim=2 * int(rng.integers(1, 9)), base=float(rng.choice([50.0, 10000.0])), **kw))
        else:
            kv = int(rng.choice([1, 2, 3]))
            dim = int(rng.integers(2, 40))
            layers.append(dl.attn_layer(heads=kv * int(rng.choice([1, 2, 4])), kv_heads=kv, dim=dim, vdim=int(rng.integers(1, 40)), scale=float(rng.choice([0.1, 0.5, 1.5])),
                                        size=int(rng.choice([1, 2, 7, 16, 33, 100, 1000])), rot_dims=2 * int(rng.integers(1, dim // 2 + 1)),
                                        base=float(rng.choice([100.0, 10000.0])),
                                        scaling={"factor": float(rng.choice([1.5, 8.0])), "original": int(rng.choice([16, 300])), "fast": 8.0, "slow": 1.0} if rng.random() < 0.7 else None,
                                        mlp=mlp))
    return dl.config(layers, vocab=int(rng.integers(2, 300)), width=int(rng.integers(3, 90)), eps=float(rng.choice([1e-6, 1e-5, 1e-3])))


@pytest.mark.parametrize("seed", range(16))
def test_sizes_drawn_at_random(seed):
    rng = np.random.default_rng(9000 + seed)
    cfg = _random_cfg(rng)
    w = dl.weights(cfg, seed=seed)
    n = int(rng.integers(20, 300))
    toks = dl.tokens(seed, n, cfg["vocab"])
    ref = do.forward(w, cfg, toks)
    m = make(cfg, w, page_tokens=int(rng.choice([4, 16, 64])))
    tl.assert_close(run_whole(m, toks), ref, "float32", cfg)
    cuts = sorted(set(int(c) for c in rng.integers(1, n, 6))) + list(range(max(1, n - 12), n))
    tl.assert_close(run_cut(m, toks, sorted(set(cuts))), ref, "float32", (cfg, cuts))
    m.close()
