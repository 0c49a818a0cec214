"""Plain, slow float64 restatement of the Duvulix design that zig_gpt2_amd/lm.py serves.

One function per mechanism, numpy only, written from the design's equations; it shares no code with the product path
(zig_gpt2_amd/ is not imported).  Weights are a dict name -> numpy array with the checkpoint's tensor names, the
configuration is the dict of config.json.

Notation: x residual stream [T, W]; u a sublayer's input; positions p count from 0 per sequence; unit(v) = v / sqrt(mean(v^2) + eps).
Every function that carries something from token to token takes what the tokens before left (None: the start of a sequence) and
returns the new one.

  n(v)   = unit(v) * (1 + w)
  x_t    = embed[token_t]
  layer  : x <- x + n_1b(mixer(n_1(x)));  x <- x + n_2b(ff(n_2(x)))            (a layer may have no ff)
  rotary : channels i and i + d/2 of the first d turn by the angle p f_i
  latent : q = W_q u per head [D plain | R rotary];  [c | k_r] = W_dkv u, c = unit(c) * w_c, k_r rotary and shared by the heads
           s_ij = scale (q_i . W_uk c_j + q^r_i . k^r_j), j <= i;  softmax;  head = sigmoid(W_g u)_h sum_j a_ij W_uv c_j;  W_o concat
           a layer that names another layer's latents reads that layer's c and k_r instead of making its own
  attention : q, k, v grouped; rotary with blended frequencies and an amplitude; keys of the query's own chunk (p // size) up to
           the query; softmax(scale q . k);  W_o concat
  mamba2 : [z | x | B | C | dt] = W_in u;  x, B, C <- silu(conv);  dt <- softplus(dt + b);  per head with its group's B, C
           S_t = exp(-exp(A) dt_t) S_(t-1) + dt_t B_t x_t^T,  y_t = S_t^T C_t + D x_t
           W_o (w * parts of (y silu(z)), every part divided by its own root mean square)
  ff     : W_down P(W_up u),  P(z) = a unit(z) + b unit(z^2) + c unit(z^3) + e
  logits = W_head n_f(x)
"""
import math

import numpy as np

F = np.float64
PROBE = None  # a list: every attention call appends (kind, softmax weights [heads, queries, keys])


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def unit(v, eps):
    return v / np.sqrt(np.mean(v * v, axis=-1, keepdims=True) + eps)


def offset_norm(w, v, eps):
    return unit(v, eps) * (1.0 + w.astype(F))


# ----------------------------------------------------------------------------------------------- rotary positions
def rotary_frequencies(rot):
    """(frequency of every pair, amplitude)."""
    d, base = int(rot["dims"]), float(rot["base"])
    f = np.array([base ** (-2.0 * i / d) for i in range(d // 2)], F)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def crossing(turns):
        return d * math.log(float(sc["original"]) / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(crossing(float(sc["fast"]))), 0)
    hi = min(math.ceil(crossing(float(sc["slow"]))), d - 1)
    ramp = np.array([min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(d // 2)], F)
    return f / float(sc["factor"]) * ramp + f * (1.0 - ramp), 0.1 * math.log(float(sc["factor"])) + 1.0


def rotate(v, positions, rot):
    """v [T, ..., channels]: the first rot['dims'] channels turned, pair (i, i + dims / 2)."""
    if not rot or int(rot["dims"]) == 0:
        return v
    d = int(rot["dims"])
    f, amp = rotary_frequencies(rot)
    a = np.asarray(positions, F)[:, None] * f[None, :]
    shape = (len(positions),) + (1,) * (v.ndim - 2) + (d // 2,)
    c, s = (np.cos(a) * amp).reshape(shape), (np.sin(a) * amp).reshape(shape)
    lo, hi = v[..., : d // 2], v[..., d // 2: d]
    return np.concatenate([lo * c - hi * s, hi * c + lo * s, v[..., d:]], axis=-1)


def softmax_rows(s):
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


# ----------------------------------------------------------------------------------------------- latent attention
def latents(w, p, m, u, positions, eps):
    """The cached part of a token: normed latent [T, kv_rank] and rotated key part [T, rot_dim]."""
    kr = int(m["kv_rank"])
    t = u @ w[p + "dkv"].astype(F).T
    return unit(t[:, :kr], eps) * w[p + "dkv.norm"].astype(F), rotate(t[:, kr:], positions, m["rot"])


def latent_attention(w, p, m, u, positions, c, k_rot):
    """c [Tk, kv_rank], k_rot [Tk, rot_dim] of positions 0 .. Tk - 1 (the queries' own included)."""
    H, D, V, R = int(m["heads"]), int(m["dim"]), int(m["vdim"]), int(m["rot_dim"])
    T, Tk = u.shape[0], c.shape[0]
    q = (u @ w[p + "q"].astype(F).T).reshape(T, H, D + R)
    q_n, q_r = q[:, :, :D], rotate(q[:, :, D:], positions, m["rot"])
    k_n = (c @ w[p + "uk"].astype(F).T).reshape(Tk, H, D)
    v = (c @ w[p + "uv"].astype(F).T).reshape(Tk, H, V)
    s = (np.einsum("ihd,jhd->hij", q_n, k_n) + np.einsum("ihd,jd->hij", q_r, k_rot)) * float(m["scale"])
    seen = np.arange(Tk)[None, :] <= np.asarray(positions)[:, None]
    a = softmax_rows(np.where(seen[None], s, -np.inf))
    if PROBE is not None:
        PROBE.append(("latent_attention", a))
    o = np.einsum("hij,jhv->ihv", a, v) * sigmoid(u @ w[p + "g"].astype(F).T)[:, :, None]
    return o.reshape(T, H * V) @ w[p + "o"].astype(F).T


# ----------------------------------------------------------------------------------------------- chunked attention
def chunk_visible(q_pos, k_pos, mask):
    """[Tq, Tk]: key at or before the query and in the query's chunk."""
    q_pos, k_pos = np.asarray(q_pos)[:, None], np.asarray(k_pos)[None, :]
    seen = k_pos <= q_pos
    if mask and int(mask["size"]) > 0:
        seen = seen & (q_pos // int(mask["size"]) == k_pos // int(mask["size"]))
    return seen


def attention(w, p, m, u, positions, cache):
    """cache: (rotated keys [T0, G, D], values [T0, G, V]) of the tokens before, or None."""
    H, G, D, V = int(m["heads"]), int(m.get("kv_heads", m["heads"])), int(m["dim"]), int(m["vdim"])
    T = u.shape[0]
    q = rotate((u @ w[p + "q"].astype(F).T).reshape(T, H, D), positions, m.get("rot"))
    k = rotate((u @ w[p + "k"].astype(F).T).reshape(T, G, D), positions, m.get("rot"))
    v = (u @ w[p + "v"].astype(F).T).reshape(T, G, V)
    if cache is not None:
        k, v = np.concatenate([cache[0], k]), np.concatenate([cache[1], v])
    s = np.einsum("ihd,jhd->hij", q, np.repeat(k, H // G, axis=1)) * float(m["scale"])
    a = softmax_rows(np.where(chunk_visible(positions, np.arange(k.shape[0]), m.get("mask"))[None], s, -np.inf))
    if PROBE is not None:
        PROBE.append(("attention", a))
    o = np.einsum("hij,jhv->ihv", a, np.repeat(v, H // G, axis=1)).reshape(T, H * V)
    return o @ w[p + "o"].astype(F).T, (k, v)


# ----------------------------------------------------------------------------------------------- state-space recurrence
def causal_conv(weight, bias, v, before):
    """weight [C, taps] (last column: the current token), v [T, C], before: the taps - 1 inputs in front (None: zeros)."""
    taps = weight.shape[1]
    if before is None:
        before = np.zeros((taps - 1, v.shape[1]), F)
    full = np.concatenate([before, v])
    out = np.stack([(full[t:t + taps] * weight.astype(F).T).sum(axis=0) + bias.astype(F) for t in range(v.shape[0])])
    return out, full[full.shape[0] - (taps - 1):] if taps > 1 else full[:0]


def ssd_recurrence(x, B, C, dt, a_log, skip, S):
    """x [T, H, V], B, C [T, H, N] (already per head), dt [T, H]; S [H, N, V] or None.  Returns (y [T, H, V], S)."""
    T, H, V = x.shape
    S = np.zeros((H, B.shape[2], V), F) if S is None else S.copy()
    y = np.zeros((T, H, V), F)
    for t in range(T):
        decay = np.exp(-np.exp(a_log) * dt[t])
        S = decay[:, None, None] * S + dt[t][:, None, None] * B[t][:, :, None] * x[t][:, None, :]
        y[t] = np.einsum("hnv,hn->hv", S, C[t]) + skip[:, None] * x[t]
    return y, S


def part_norm(w, v, parts, eps):
    T, n = v.shape
    return unit(v.reshape(T, parts, n // parts), eps).reshape(T, n) * w.astype(F)


def mamba2(w, p, m, u, state, eps):
    H, V, N, G = int(m["heads"]), int(m["vdim"]), int(m["state"]), int(m["groups"])
    T, inner = u.shape[0], H * V
    before, S = state if state is not None else (None, None)
    t = u @ w[p + "in"].astype(F).T
    z, xbc, dt = t[:, :inner], t[:, inner:2 * inner + 2 * G * N], t[:, 2 * inner + 2 * G * N:]
    xbc, before = causal_conv(w[p + "conv"], w[p + "conv.b"], xbc, before)
    xbc = silu(xbc)
    x = xbc[:, :inner].reshape(T, H, V)
    B = np.repeat(xbc[:, inner:inner + G * N].reshape(T, G, N), H // G, axis=1)
    C = np.repeat(xbc[:, inner + G * N:].reshape(T, G, N), H // G, axis=1)
    dt = softplus(dt + w[p + "dt_bias"].astype(F))
    y, S = ssd_recurrence(x, B, C, dt, w[p + "A_log"].astype(F), w[p + "D"].astype(F), S)
    y = part_norm(w[p + "norm"], y.reshape(T, inner) * silu(z), int(m["norm_groups"]), eps)
    return y @ w[p + "o"].astype(F).T, (before, S)


# ----------------------------------------------------------------------------------------------- feed-forward
def polynorm(act, z, eps):
    a, b, c, e = (float(v) for v in np.asarray(act).reshape(-1))
    return a * unit(z, eps) + b * unit(z ** 2, eps) + c * unit(z ** 3, eps) + e


def dense_ff(w, p, u, eps):
    return polynorm(w[p + "act"], u @ w[p + "up"].astype(F).T, eps) @ w[p + "down"].astype(F).T


# ----------------------------------------------------------------------------------------------- the stack
class Sequence:
    """What a sequence carries between calls: per layer the recurrent state or the cached keys, and the token count."""

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
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        u = offset_norm(w[p + "norm1"], x, eps)
        if layer["type"] == "latent_attention":
            src = m.get("kv_from")
            if src is None:
                new = latents(w, p + "mix.", m, u, positions, eps)
                old = seq.state[i]
                seq.state[i] = new if old is None else tuple(np.concatenate([a, b]) for a, b in zip(old, new))
            y = latent_attention(w, p + "mix.", m, u, positions, *seq.state[i if src is None else int(src)])
        elif layer["type"] == "attention":
            y, seq.state[i] = attention(w, p + "mix.", m, u, positions, seq.state[i])
        elif layer["type"] == "mamba2":
            y, seq.state[i] = mamba2(w, p + "mix.", m, u, seq.state[i], eps)
        else:
            raise ValueError(layer["type"])
        x = x + offset_norm(w[p + "norm1b"], y, eps)
        if layer.get("mlp"):
            y = dense_ff(w, p + "mlp.", offset_norm(w[p + "norm2"], x, eps), eps)
            x = x + offset_norm(w[p + "norm2b"], y, eps)
        if trace is not None:
            trace.append(x.copy())
    seq.n += len(tokens)
    return offset_norm(w["final.norm"], x, eps) @ w["head"].astype(F).T


def generate(w, cfg, prompt, n_new):
    seq = Sequence(cfg)
    out, logits = [], forward(w, cfg, prompt, seq)
    for _ in range(n_new):
        out.append(int(np.argmax(logits[-1])))
        logits = forward(w, cfg, [out[-1]], seq)
    return out
