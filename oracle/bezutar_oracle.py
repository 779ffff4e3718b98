"""Plain restatement of the Bezutar design on the CPU: slow, one function per mechanism, no code shared with the product.

float64 numpy, whole sequences at once, no cache: the logits of a sequence are a function of its token ids alone, so portions, batches, pages, state
slots and decode steps are all compared against the same numbers.  Weights are a dict of float arrays under the checkpoint's tensor names."""
from __future__ import annotations

import math

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def softplus(z):
    return np.logaddexp(0.0, z)


def silu(z):
    return z * sigmoid(z)


def unit_rms(x, eps):
    """x over its root mean square along the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def zero_centred_norm(x, w, eps):
    """RMS norm whose stored weight is the difference from one."""
    return unit_rms(x, eps) * (1.0 + w)


# ------------------------------------------------------------------ embedding
def bigram_rows(ids, buckets, mul_prev, mul_cur):
    """Row of the bigram table for every token; a sequence's first token has no predecessor and takes the row behind the buckets."""
    rows = [buckets]
    for prev, cur in zip(ids[:-1], ids[1:]):
        rows.append((int(prev) * mul_prev + int(cur) * mul_cur) % buckets)
    return rows


def embed(cfg, w, ids):
    b = cfg["embedding"]["bigram"]
    rows = bigram_rows(list(ids), w["bigram"].shape[0] - 1, b["mul_prev"], b["mul_cur"])
    return w["embed"][np.asarray(ids)] + w["bigram"][rows] + w["pos"][:len(ids)]


# ------------------------------------------------------------------ what surrounds a sublayer
def causal_conv(h, w):
    """h [n, W] plus a causal filter over time per channel: tap j of w [W, taps] reads taps - 1 - j tokens back."""
    taps, out = w.shape[1], h.copy()
    for back in range(taps):
        shifted = np.zeros_like(h)
        shifted[back:] = h[:max(len(h) - back, 0)]
        out = out + shifted * w[:, taps - 1 - back]
    return out


def streams_in(x, w, p):
    """x [streams, n, W] -> what the sublayer's norm reads."""
    return np.tensordot(w[p + "in"], x, axes=1)


def streams_out(x, y, w, p):
    """Every stream anew from all old ones and the sublayer's output; mix is indexed [from, to]."""
    return np.stack([np.tensordot(w[p + "mix"][:, t], x, axes=1) + w[p + "out"][t] * y for t in range(x.shape[0])])


# ------------------------------------------------------------------ mLSTM
def mlstm_recurrence(q, k, v, i, f, state=None):
    """q, k [n, heads, dim], v [n, heads, vdim], log gates i, f [n, heads].  Returns o [n, heads, vdim] and (S, norm vector, running maximum)."""
    n, H, D = q.shape
    if state is None:
        S, z, m = np.zeros((H, D, v.shape[2])), np.zeros((H, D)), np.zeros(H)
    else:
        S, z, m = (a.copy() for a in state)
    o = np.empty_like(v)
    for t in range(n):
        new = np.maximum(f[t] + m, i[t])
        keep, add = np.exp(f[t] + m - new), np.exp(i[t] - new)
        S = keep[:, None, None] * S + add[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        z = keep[:, None] * z + add[:, None] * k[t]
        m = new
        below = np.maximum(np.abs(np.sum(z * q[t], axis=1)), np.exp(-m)) + 1e-6
        o[t] = np.einsum("hde,hd->he", S, q[t]) / below[:, None]
    return o, (S, z, m)


def capped(z, cap):
    return cap * np.tanh(z / cap)


def mlstm(h, w, p, mx, eps):
    n, H, D, V, cap = h.shape[0], mx["heads"], mx["dim"], mx["vdim"], mx["gate_cap"]
    q = (h @ w[p + "q"].T).reshape(n, H, D) * D ** -0.5
    k, v = (h @ w[p + "k"].T).reshape(n, H, D), (h @ w[p + "v"].T).reshape(n, H, V)
    i = capped(h @ w[p + "i"].T + w[p + "i.b"], cap)
    f = -softplus(-capped(h @ w[p + "f"].T + w[p + "f.b"], cap))
    o, _ = mlstm_recurrence(q, k, v, i, f)
    return (unit_rms(o, eps).reshape(n, H * V) * w[p + "norm"] * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


# ------------------------------------------------------------------ minGRU
def mingru_recurrence(z, u, state=None):
    """Update gate z and pre-activation u [n, width]."""
    cand = np.where(u >= 0, u + 0.5, sigmoid(u))
    S = np.zeros(z.shape[1]) if state is None else state.copy()
    out = np.empty_like(z)
    for t in range(len(z)):
        S = (1.0 - z[t]) * S + z[t] * cand[t]
        out[t] = S
    return out, S


def mingru(h, w, p):
    S, _ = mingru_recurrence(sigmoid(h @ w[p + "z"].T + w[p + "z.b"]), h @ w[p + "x"].T + w[p + "x.b"])
    return (S * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


# ------------------------------------------------------------------ latent attention
def rotary_frequencies(dims, base, scaling=None):
    """(one frequency per pair, the factor on cos and sin).  scaling: YaRN's dict or None."""
    i = np.arange(dims // 2, dtype=np.float64)
    f = np.power(float(base), -2.0 * i / dims)
    if not scaling:
        return f, 1.0

    def turns(t):   # the (fractional) pair that makes t turns over the original context
        return dims * math.log(scaling["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(turns(scaling["fast"])), 0), min(math.ceil(turns(scaling["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / scaling["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(scaling["factor"]) + 1.0


def rotate_halves(x, positions, rot):
    """x [n, ..., d]: number i turns with number i + dims / 2; what lies behind dims stays."""
    f, gain = rotary_frequencies(rot["dims"], rot["base"], rot.get("scaling"))
    n = len(f)
    a = positions.reshape((-1,) + (1,) * (x.ndim - 1)) * f
    c, s = np.cos(a) * gain, np.sin(a) * gain
    u, v, out = x[..., :n], x[..., n:2 * n], x.copy()
    out[..., :n], out[..., n:2 * n] = u * c - v * s, v * c + u * s
    return out


def sink_softmax(s, mask, sink):
    """exp(s) / (exp(sink) + sum exp(s)) over the masked-in entries."""
    s = np.where(mask, s, -np.inf)
    m = np.maximum(s.max(axis=-1, keepdims=True), sink)
    p = np.exp(s - m)
    return p / (np.exp(sink - m) + p.sum(axis=-1, keepdims=True))


def latents(h, w, p, mx, eps):
    """What a layer caches: the normed latent [n, kv_rank] and the rotated key part [n, rot_dim] that all heads share."""
    y = h @ w[p + "dkv"].T
    R = mx["kv_rank"]
    return unit_rms(y[:, :R], eps) * w[p + "dkv.norm"], rotate_halves(y[:, R:], np.arange(len(h), dtype=np.float64), mx["rot"])


def latent_attention(h, w, p, mx, cached, eps):
    n, H, D, T, V = h.shape[0], mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"]
    c, k_rot = cached
    q = ((unit_rms(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]) @ w[p + "uq"].T).reshape(n, H, D + T)
    q_rot = rotate_halves(q[:, :, D:], np.arange(n, dtype=np.float64), mx["rot"])
    k, v = (c @ w[p + "uk"].T).reshape(n, H, D), (c @ w[p + "uv"].T).reshape(n, H, V)
    gate, mask = sigmoid(h @ w[p + "g"].T), np.tril(np.ones((n, n), dtype=bool))
    out = np.empty((n, H, V))
    for a in range(H):
        s = (q[:, a, :D] @ k[:, a].T + q_rot[:, a] @ k_rot.T) * mx["scale"]
        out[:, a] = sink_softmax(s, mask, w[p + "sink"][a]) @ v[:, a] * gate[:, a:a + 1]
    return out.reshape(n, H * V) @ w[p + "o"].T


# ------------------------------------------------------------------ feed-forward
def xielu(z, p, q):
    return np.where(z > 0, softplus(p) * z * z + 0.5 * z, (0.5 + softplus(q)) * (np.expm1(np.minimum(z, 0.0)) - z) + 0.5 * z)


def dense(h, w, p):
    return xielu(h @ w[p + "up"].T, *w[p + "act"]) @ w[p + "down"].T


# ------------------------------------------------------------------ the model
def forward(cfg, w, ids, layers_out=None):
    """Logits [n, vocab] of one sequence; layers_out (a list) receives the sum of the streams after every layer."""
    eps = cfg["norm"]["eps"]
    x = np.stack([embed(cfg, w, ids)] * cfg["streams"])
    cached = {}
    for i, lay in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", lay["mixer"]
        h = causal_conv(zero_centred_norm(streams_in(x, w, p + "hc1."), w[p + "norm1"], eps), w[p + "canon1"])
        if lay["type"] == "mlstm":
            y = mlstm(h, w, p + "mix.", mx, eps)
        elif lay["type"] == "mingru":
            y = mingru(h, w, p + "mix.")
        else:
            j = mx.get("kv_from")
            cached[i] = cached[j] if j is not None else latents(h, w, p + "mix.", mx, eps)
            y = latent_attention(h, w, p + "mix.", mx, cached[i], eps)
        x = streams_out(x, y, w, p + "hc1.")
        if lay.get("mlp") is not None:
            y = dense(zero_centred_norm(streams_in(x, w, p + "hc2."), w[p + "norm2"], eps), w, p + "mlp.")
            x = streams_out(x, y, w, p + "hc2.")
        if layers_out is not None:
            layers_out.append(x.sum(axis=0))
    return zero_centred_norm(x.sum(axis=0), w["final.norm"], eps) @ w["head"].T
