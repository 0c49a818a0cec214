"""Small random Duvulix configurations and weights for the tests (bf16-representable values, so that the float64 oracle and the
bf16-storage device path see the same numbers)."""
import numpy as np

from zig_gpt2_amd.synth import round_bf16  # noqa: F401  (also for the tests that build weights by hand)


def mamba_layer(heads=4, vdim=10, state=12, groups=2, conv=3, norm_groups=1, mlp=None):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}, "mlp": mlp}


def latent_layer(heads=3, dim=10, vdim=14, rot_dim=6, kv_rank=20, scale=0.25, base=5000.0, kv_from=None, mlp=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "rot_dim": rot_dim, "kv_rank": kv_rank, "scale": scale, "rot": {"base": base, "dims": rot_dim}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def attn_layer(heads=4, kv_heads=2, dim=12, vdim=8, scale=0.3, size=9, rot_dims=None, base=1000.0, scaling="default", mlp=None):
    if scaling == "default":
        scaling = {"factor": 6.0, "original": 96, "fast": 12.0, "slow": 1.5}
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    d = dim if rot_dims is None else rot_dims
    if d:
        m["rot"] = {"base": base, "dims": d}
        if scaling:
            m["rot"]["scaling"] = scaling
    if size:
        m["mask"] = {"size": size}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def dense(ff=28):
    return {"kind": "dense", "ff": ff}


def config(layers, vocab=89, width=40, eps=1e-5):
    return {"architecture": "Duvulix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


def weights(cfg, seed=0, rate=(0.5, 8.0), dt_bias=(-1.5, 1.0), embed_std=1.0):
    """Random tensors for every name of the configuration.  Matrices ~ N(0, 1 / fan_in); rate: range of exp(A_log); dt_bias: mean and
    deviation of the step sizes' bias."""
    from zig_gpt2_amd import lm

    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in sorted(lm.LMConfig.from_json(cfg).tensor_shapes().items()):
        leaf = name.split(".")[-1]
        if name == "embed":
            a = rng.normal(0.0, embed_std, shape)
        elif leaf == "A_log":
            a = np.log(rng.uniform(rate[0], rate[1], shape))
        elif leaf == "dt_bias":
            a = rng.normal(dt_bias[0], dt_bias[1], shape)
        elif leaf == "act":
            a = np.array([0.8, -0.4, 0.3, 0.15]) + rng.normal(0.0, 0.1, shape)
        elif leaf == "conv":
            a = rng.normal(0.0, 0.6, shape)
        elif leaf == "b":
            a = rng.normal(0.0, 0.2, shape)
        elif len(shape) == 2:
            a = rng.normal(0.0, 1.0 / np.sqrt(shape[1]), shape)
        elif leaf == "D" or name.endswith("mix.norm") or name.endswith("dkv.norm"):
            a = 1.0 + rng.normal(0.0, 0.2, shape)
        else:  # norm offsets around zero
            a = rng.normal(0.0, 0.1, shape)
        out[name] = round_bf16(np.asarray(a, np.float32)).reshape(shape)
    return out


def tokens(seed, n, vocab):
    return np.random.default_rng(6000 + seed).integers(0, vocab, n).astype(np.int32)
