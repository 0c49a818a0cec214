"""Plain, slow float64 restatement of the Pemuvik design that zig_gpt2_amd/lm.py serves.

One function per mechanism, numpy only, written from the design's equations; it shares no code with the product path
(zig_gpt2_amd/ is not imported).  Weights are a dict name -> numpy array with the checkpoint's tensor names, the
configuration is the dict of config.json.

Notation: x residual stream [T, W]; u a sublayer's input; positions p count from 0 per sequence; unit(v) = v / sqrt(mean(v^2) + eps).
Every function that carries something from token to token takes what the tokens before left (None: the start of a sequence) and
returns the new one.

  n(v)   = unit(v) * w
  x_t    = embed[token_t]
  layer  : x <- x + ls1 * mixer(n_1(x)) + ls2 * ff(n_2(x))         (both sublayers read the same x; a layer may have no ff)
  rotary : channels 2i and 2i + 1 of the first d turn by the angle p base^(-2i/d)
  latent : q = W_q u per head [D plain | R rotary];  [c | k_r] = W_dkv u, c = unit(c) * w_c, k_r rotary and shared by the heads
           s_ij = scale (q_i . W_uk c_j + q^r_i . k^r_j), j <= i;  a_ij = exp(s_ij) / (exp(sink_h) + sum_j exp(s_ij))
           W_o concat_h(sum_j a_ij W_uv c_j)
  gate attention : q, k, v = W u + b grouped; q, k rotary; v <- unit(v) per head; in a layer that mixes values
           v <- (1 - l) v + l v', v' the first such layer's v of the same token
           a_ij = sigmoid(scale q_i . k_j + pb_h) for 0 <= i - j < size (no sum over keys);  W_o concat_h(sum_j a_ij v_j) + b_o
  dense  : W_down (gelu(W_gate u) * W_up u), gelu by its tanh form
  experts: s = softmax(W_r u); r = s + correction; the outputs are cut into groups of neighbours, a group ranks by its largest r, only
           the best groups stay; the `top` largest r of those; weights s / (sum of the chosen s + 1e-20)
           the last `identity` outputs stand for u itself; the others are W_down(silu(W_gate u) * W_up u)
           + sigmoid(w_sg . u) * the expert every token uses
  logits = embed . n_f(x)
"""
import math

import numpy as np

F = np.float64
PROBE = None  # a list: every attention call appends (kind, weights [heads, queries, keys]); every router call ("router", picks, weights)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def unit(v, eps):
    return v / np.sqrt(np.mean(v * v, axis=-1, keepdims=True) + eps)


def norm(w, v, eps):
    return unit(v, eps) * w.astype(F)


def linear(w, name, u):
    """W u, plus the bias where the projection has one."""
    y = u @ w[name].astype(F).T
    return y + w[name + ".b"].astype(F) if name + ".b" in w else y


# ----------------------------------------------------------------------------------------------- rotary positions
def rotate(v, positions, rot):
    """v [T, ..., channels]: the first rot['dims'] channels turned in neighbouring pairs; the rest pass."""
    d = int(rot["dims"]) if rot else 0
    if d == 0:
        return v
    f = float(rot["base"]) ** (-2.0 * np.arange(d // 2) / d)
    a = (np.asarray(positions, F)[:, None] * f).reshape((len(positions),) + (1,) * (v.ndim - 2) + (d // 2,))
    out = v.copy()
    out[..., 0:d:2] = v[..., 0:d:2] * np.cos(a) - v[..., 1:d:2] * np.sin(a)
    out[..., 1:d:2] = v[..., 1:d:2] * np.cos(a) + v[..., 0:d:2] * np.sin(a)
    return out


# ----------------------------------------------------------------------------------------------- latent attention with a sink
def latents(w, p, m, u, positions, eps):
    """The cached part of a token: normed latent [T, kv_rank] and rotated key part [T, rot_dim]."""
    kr = int(m["kv_rank"])
    t = linear(w, p + "dkv", u)
    return norm(w[p + "dkv.norm"], t[:, :kr], eps), rotate(t[:, kr:], positions, m["rot"])


def sink_softmax(s, sink):
    """s [H, queries, keys] with -inf for keys out of sight; the sink adds to the denominator only."""
    top = np.maximum(s.max(axis=-1, keepdims=True), sink[:, None, None])
    e = np.exp(s - top)
    return e / (e.sum(axis=-1, keepdims=True) + np.exp(sink[:, None, None] - top))


def latent_attention(w, p, m, u, positions, c, k_rot):
    """c [Tk, kv_rank], k_rot [Tk, rot_dim] of positions 0 .. Tk - 1 (the queries' own included)."""
    H, D, V, R = int(m["heads"]), int(m["dim"]), int(m["vdim"]), int(m["rot_dim"])
    T, Tk = u.shape[0], c.shape[0]
    q = linear(w, p + "q", u).reshape(T, H, D + R)
    q_n, q_r = q[:, :, :D], rotate(q[:, :, D:], positions, m["rot"])
    k_n, v = linear(w, p + "uk", c).reshape(Tk, H, D), linear(w, p + "uv", c).reshape(Tk, H, V)
    s = (np.einsum("ihd,jhd->hij", q_n, k_n) + np.einsum("ihd,jd->hij", q_r, k_rot)) * float(m["scale"])
    seen = np.arange(Tk)[None, :] <= np.asarray(positions)[:, None]
    a = sink_softmax(np.where(seen[None], s, -np.inf), w[p + "sink"].astype(F))
    if PROBE is not None:
        PROBE.append(("latent_attention", a))
    return linear(w, p + "o", np.einsum("hij,jhv->ihv", a, v).reshape(T, H * V))


# ----------------------------------------------------------------------------------------------- windowed attention with sigmoid weights
def window_visible(q_pos, k_pos, mask):
    """[Tq, Tk]: key at or before the query and, with a mask, fewer than its size positions back."""
    dist = np.asarray(q_pos)[:, None] - np.asarray(k_pos)[None, :]
    seen = dist >= 0
    if mask and int(mask.get("size") or 0) > 0:
        seen = seen & (dist < int(mask["size"]))
    return seen


def mix_values(v, lam, v_first):
    return (1.0 - lam) * v + lam * v_first


def gate_attention(w, p, m, u, positions, eps, cache, v_first):
    """cache: (rotated keys [T0, G, D], values [T0, G, V]) of the tokens before, or None.  v_first: the values of the first layer that
    mixes (None in that layer).  Returns (out, cache, the layer's values of these tokens in front of the mix)."""
    H, G, D, V = int(m["heads"]), int(m.get("kv_heads", m["heads"])), int(m["dim"]), int(m["vdim"])
    T = u.shape[0]
    q = rotate(linear(w, p + "q", u).reshape(T, H, D), positions, m.get("rot"))
    k = rotate(linear(w, p + "k", u).reshape(T, G, D), positions, m.get("rot"))
    own = v = unit(linear(w, p + "v", u).reshape(T, G, V), eps)
    if m.get("v_mix") and v_first is not None:
        v = mix_values(v, float(np.asarray(w[p + "vmix"]).reshape(-1)[0]), v_first)
    if cache is not None:
        k, v = np.concatenate([cache[0], k]), np.concatenate([cache[1], v])
    s = np.einsum("ihd,jhd->hij", q, np.repeat(k, H // G, axis=1)) * float(m["scale"]) + w[p + "pb"].astype(F)[:, None, None]
    a = np.where(window_visible(positions, np.arange(k.shape[0]), m.get("mask"))[None], sigmoid(s), 0.0)
    if PROBE is not None:
        PROBE.append(("attention", a))
    o = np.einsum("hij,jhv->ihv", a, np.repeat(v, H // G, axis=1)).reshape(T, H * V)
    return linear(w, p + "o", o), (k, v), own


# ----------------------------------------------------------------------------------------------- feed-forward
def gated_unit(w, p, u, act):
    return linear(w, p + "down", act(linear(w, p + "gate", u)) * linear(w, p + "up", u))


def route(z, correction, top, groups):
    """z [T, N] logits -> (chosen outputs [T, top], their weights).  groups: {count, keep} or None."""
    e = np.exp(z - z.max(axis=-1, keepdims=True))
    s = e / e.sum(axis=-1, keepdims=True)
    r = s + correction
    T, N = z.shape
    if groups and int(groups["count"]) > 1:
        n, keep = int(groups["count"]), int(groups["keep"])
        rank = r.reshape(T, n, N // n).max(axis=-1)
        best = np.argsort(-rank, axis=-1, kind="stable")[:, :keep]
        stays = np.zeros((T, n), bool)
        np.put_along_axis(stays, best, True, axis=-1)
        r = np.where(np.repeat(stays, N // n, axis=-1), r, -np.inf)
    pick = np.argsort(-r, axis=-1, kind="stable")[:, :top]
    wt = np.take_along_axis(s, pick, axis=-1)
    return pick, wt / (wt.sum(axis=-1, keepdims=True) + 1e-20)


def experts(w, p, mlp, u):
    r = mlp["router"]
    E = int(r["experts"])
    pick, wt = route(u @ w[p + "router"].astype(F).T, w[p + "correction"].astype(F), int(r["top"]), r.get("groups"))
    if PROBE is not None:
        PROBE.append(("router", pick, wt))
    y = np.zeros_like(u)
    for t in range(u.shape[0]):
        for e, a in zip(pick[t], wt[t]):
            y[t] += a * (gated_unit(w, f"{p}e{e}.", u[t:t + 1], silu)[0] if e < E else u[t])
    if mlp.get("shared"):
        y = y + sigmoid(linear(w, p + "shared.sg", u)) * gated_unit(w, p + "shared.", u, silu)
    return y


def feed_forward(w, p, mlp, u):
    return gated_unit(w, p, u, gelu_tanh) if mlp["kind"] == "dense" else experts(w, p, mlp, u)


# ----------------------------------------------------------------------------------------------- the stack
class Sequence:
    """What a sequence carries between calls: per layer the cached keys and values or latents, and the token count."""

    def __init__(self, cfg):
        self.state = [None] * len(cfg["layers"])
        self.n = 0


def forward(w, cfg, tokens, seq=None, trace=None):
    """Logits [T, vocab] of the next `tokens` of a sequence (seq: a Sequence that is moved on; None: a new one).
    trace: a list that receives the residual stream behind every layer."""
    seq = seq or Sequence(cfg)
    eps = float(cfg["norm"]["eps"])
    positions = np.arange(seq.n, seq.n + len(tokens))
    x = w["embed"].astype(F)[np.asarray(tokens)]
    v_first = None
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        u = norm(w[p + "norm1"], x, eps)
        if layer["type"] == "latent_attention":
            new = latents(w, p + "mix.", m, u, positions, eps)
            old = seq.state[i]
            seq.state[i] = new if old is None else tuple(np.concatenate([a, b]) for a, b in zip(old, new))
            y = latent_attention(w, p + "mix.", m, u, positions, *seq.state[i])
        elif layer["type"] == "attention":
            y, seq.state[i], own = gate_attention(w, p + "mix.", m, u, positions, eps, seq.state[i], v_first)
            if m.get("v_mix") and v_first is None:
                v_first = own
        else:
            raise ValueError(layer["type"])
        y = w[p + "ls1"].astype(F) * y
        if layer.get("mlp"):
            y = y + w[p + "ls2"].astype(F) * feed_forward(w, p + "mlp.", layer["mlp"], norm(w[p + "norm2"], x, eps))
        x = x + y
        if trace is not None:
            trace.append(x.copy())
    seq.n += len(tokens)
    return norm(w["final.norm"], x, eps) @ w["embed"].astype(F).T


def generate(w, cfg, prompt, n_new):
    seq = Sequence(cfg)
    out, logits = [], forward(w, cfg, prompt, seq)
    for _ in range(n_new):
        out.append(int(np.argmax(logits[-1])))
        logits = forward(w, cfg, [out[-1]], seq)
    return out
