"""Plain restatement of the Kodupel design on the CPU: slow, one function per mechanism, no code shared with the product.

float64 numpy, whole sequences at once, no cache: the logits of a sequence are a function of its token ids alone, so portions, batches, pages, state
slots and decode steps are all compared against the same numbers.  Weights are a dict of float arrays under the checkpoint's tensor names."""
from __future__ import annotations

import math

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def unit_rms(x, eps):
    """x over its root mean square along the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def zero_centred_norm(x, w, eps):
    """RMS norm whose stored weight is the difference from one."""
    return unit_rms(x, eps) * (1.0 + w)


# ------------------------------------------------------------------ rotation
def rotary_frequencies(dims, base, scaling=None):
    """(one frequency per pair, the factor on cos and sin).  scaling: YaRN's dict or None."""
    i = np.arange(dims // 2, dtype=np.float64)
    f = np.power(float(base), -2.0 * i / dims)
    if not scaling:
        return f, 1.0

    def turns(t):   # the (fractional) pair-dimension that makes t turns over the original context
        return dims * math.log(scaling["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(turns(scaling["fast"])), 0), min(math.ceil(turns(scaling["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / scaling["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(scaling["factor"]) + 1.0


def rotate_pairs(x, positions, freqs, gain):
    """x [n, heads, dim]: neighbours (2 i, 2 i + 1) turn by position * freqs[i]; what lies behind the last pair stays."""
    out = x.copy()
    a = positions[:, None, None] * freqs
    c, s = np.cos(a) * gain, np.sin(a) * gain
    n = 2 * len(freqs)
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out[..., 0:n:2], out[..., 1:n:2] = u * c - v * s, v * c + u * s
    return out


# ------------------------------------------------------------------ softmax attention
def sink_softmax(s, mask):
    """exp(s) / (1 + sum exp(s)) over the masked-in entries: one more score of 0 that has no value."""
    s = np.where(mask, s, -np.inf)
    m = np.maximum(s.max(axis=-1, keepdims=True), 0.0)
    p = np.exp(s - m)
    return p / (np.exp(-m) + p.sum(axis=-1, keepdims=True))


def keys_values(h, w, p, mx, eps):
    """What a layer caches: keys [n, G, dim] after norm and rotation, values [n, G, vdim] over their root mean square."""
    n, G = h.shape[0], mx["kv_heads"]
    k = (h @ w[p + "k"].T + w[p + "k.b"]).reshape(n, G, mx["dim"])
    v = (h @ w[p + "v"].T + w[p + "v.b"]).reshape(n, G, mx["vdim"])
    k = unit_rms(k, eps) * w[p + "k.norm"]
    rot = mx["rot"]
    k = rotate_pairs(k, np.arange(n, dtype=np.float64), *rotary_frequencies(rot["dims"], rot["base"], rot.get("scaling")))
    return k, unit_rms(v, eps)


def attention(h, w, p, mx, kv, eps):
    n, H, G, rot = h.shape[0], mx["heads"], mx["kv_heads"], mx["rot"]
    k, v = kv
    q = (h @ w[p + "q"].T + w[p + "q.b"]).reshape(n, H, mx["dim"])
    q = unit_rms(q, eps) * w[p + "q.norm"]
    q = rotate_pairs(q, np.arange(n, dtype=np.float64), *rotary_frequencies(rot["dims"], rot["base"], rot.get("scaling")))
    gate = sigmoid(h @ w[p + "g"].T)
    mask = np.tril(np.ones((n, n), dtype=bool))
    out = np.empty((n, H, mx["vdim"]))
    for a in range(H):
        b = a // (H // G)
        out[:, a] = sink_softmax((q[:, a] @ k[:, b].T) * mx["scale"], mask) @ v[:, b] * gate[:, a:a + 1]
    return out.reshape(n, -1) @ w[p + "o"].T + w[p + "o.b"]


# ------------------------------------------------------------------ generalised delta rule
def delta_decay(h, w, p):
    return np.exp(-math.exp(-0.5) * sigmoid(np.tanh(h @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"]))


def delta_recurrence(r, k, v, decay, rate, state=None):
    """All [n, heads, dim].  Returns o [n, heads, dim] and the state [heads, dim (key), dim (value)] behind the last token."""
    n, H, D = r.shape
    S = np.zeros((H, D, D)) if state is None else state.copy()
    u = k / np.sqrt(np.sum(k * k, axis=-1, keepdims=True) + 1e-6)
    o = np.empty((n, H, D))
    for t in range(n):
        seen = np.einsum("hd,hde->he", u[t], S)
        S = decay[t][:, :, None] * S - (rate[t] * u[t])[:, :, None] * seen[:, None, :] + k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hde,hd->he", S, r[t])
    return o, S


def general_delta(h, w, p, mx, eps):
    n, H, D = h.shape[0], mx["heads"], mx["dim"]

    def heads(y):
        return y.reshape(n, H, D)
    rate = sigmoid(h @ w[p + "a"].T + w[p + "a.b"])
    o, _ = delta_recurrence(heads(h @ w[p + "r"].T), heads(h @ w[p + "k"].T), heads(h @ w[p + "v"].T), heads(delta_decay(h, w, p)), heads(rate))
    return (unit_rms(o, eps).reshape(n, H * D) * w[p + "norm"] * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


# ------------------------------------------------------------------ experts
def clipped_expert(h, w, p, limit):
    g, u = np.minimum(h @ w[p + "gate"].T, limit), np.clip(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def choose_experts(h, w, p, top):
    """([n, top] expert numbers, [n, top] their weights, [n] how far the last chosen is ahead of the first that is not): the choice counts the correction,
    the weights do not."""
    s = sigmoid(h @ w[p + "router"].T)
    counted = s + w[p + "correction"]
    order = np.argsort(-counted, axis=-1, kind="stable")
    best, ranked = order[:, :top], np.take_along_axis(counted, order, axis=-1)
    lead = ranked[:, top - 1] - ranked[:, top] if top < s.shape[-1] else np.full(len(s), np.inf)
    return best, np.take_along_axis(s, best, axis=-1), lead


def mixture(h, w, p, ff, leads=None):
    best, weight, lead = choose_experts(h, w, p, ff["router"]["top"])
    if leads is not None:
        leads.append(lead)
    y = np.zeros_like(h)
    for e in range(ff["router"]["experts"]):
        row, slot = np.nonzero(best == e)
        if len(row):
            y[row] += weight[row, slot][:, None] * clipped_expert(h[row], w, f"{p}e{e}.", ff["expert"]["limit"])
    return y


# ------------------------------------------------------------------ the model
def forward(cfg, w, ids, layers_out=None, leads=None):
    """Logits [n, vocab] of one sequence; layers_out (a list) receives the residual stream after every layer, leads every mixture's closest calls."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][np.asarray(ids)] * cfg["embedding"]["scale"]
    cached = {}
    for i, lay in enumerate(cfg["layers"]):
        p, mx, ff = f"l{i}.", lay["mixer"], lay.get("mlp")
        if lay["type"] == "general_delta":
            y = general_delta(x, w, p + "mix.", mx, eps)
        else:
            j = mx.get("kv_from")
            cached[i] = cached[j] if j is not None else keys_values(x, w, p + "mix.", mx, eps)
            y = attention(x, w, p + "mix.", mx, cached[i], eps)
        x = x + zero_centred_norm(y, w[p + "norm1"], eps)
        if ff is not None:
            x = x + zero_centred_norm(mixture(x, w, p + "mlp.", ff, leads), w[p + "norm2"], eps)
        if layers_out is not None:
            layers_out.append(x.copy())
    return zero_centred_norm(x, w["final.norm"], eps) @ w["head"].T
