"""Small random Pemuvik configurations and weights for the tests (bf16-representable values, so that the float64 oracle and the
bf16-storage device path see the same numbers)."""
import numpy as np

from zig_gpt2_amd.synth import round_bf16  # noqa: F401  (also for the tests that build weights by hand)


def latent_layer(heads=3, dim=10, vdim=14, rot_dim=6, kv_rank=20, scale=0.3, base=3000.0, mlp=None):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "rot_dim": rot_dim, "kv_rank": kv_rank, "scale": scale,
                                                  "rot": {"base": base, "dims": rot_dim}}, "mlp": mlp}


def attn_layer(heads=4, kv_heads=2, dim=12, vdim=8, scale=0.4, size=9, rot_dims=6, base=1000.0, v_mix=True, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if rot_dims:
        m["rot"] = {"base": base, "dims": rot_dims}
    if size:
        m["mask"] = {"size": size}
    if v_mix:
        m["v_mix"] = True
    return {"type": "attention", "mixer": m, "mlp": mlp}


def dense(ff=28):
    return {"kind": "dense", "ff": ff}


def moe(ff=10, experts=6, identity=2, groups=(4, 2), top=3, shared=18):
    r = {"experts": experts, "top": top}
    if groups and groups[0] > 1:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    if identity:
        r["identity"] = identity
    out = {"kind": "moe", "expert": {"ff": ff}, "router": r}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def config(layers, vocab=89, width=40, eps=1e-5):
    return {"architecture": "Pemuvik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


def weights(cfg, seed=0, embed_std=1.0, router_std=1.0):
    """Random tensors for every name of the configuration.  Matrices ~ N(0, 1 / fan_in), the router's times router_std."""
    from zig_gpt2_amd import lm

    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in sorted(lm.LMConfig.from_json(cfg).tensor_shapes().items()):
        leaf = name.split(".")[-1]
        if name == "embed":
            a = rng.normal(0.0, embed_std, shape)
        elif leaf == "router":
            a = rng.normal(0.0, router_std / np.sqrt(shape[1]), shape)
        elif leaf == "correction":  # of the size of the scores: some choices become negative
            a = rng.normal(0.0, 0.15, shape)
        elif leaf == "pb":
            a = rng.normal(-1.0, 0.8, shape)
        elif leaf == "sink":
            a = rng.normal(0.5, 1.0, shape)
        elif leaf == "vmix":
            a = np.asarray(rng.uniform(0.2, 0.8))
        elif leaf == "b":
            a = rng.normal(0.0, 0.3, shape)
        elif len(shape) == 2:
            a = rng.normal(0.0, 1.0 / np.sqrt(shape[1]), shape)
        elif leaf in ("ls1", "ls2"):
            a = rng.normal(0.6, 0.3, shape)
        else:  # norm weights around one
            a = 1.0 + rng.normal(0.0, 0.2, shape)
        out[name] = round_bf16(np.asarray(a, np.float32)).reshape(shape)
    return out


def tokens(seed, n, vocab):
    return np.random.default_rng(7000 + seed).integers(0, vocab, n).astype(np.int32)
