"""Plain restatement of the Lagelorn design on the CPU: slow, one function per mechanism, no code shared with the product.

float64 numpy, whole sequences at once, no cache: the logits of a sequence are a function of its token ids alone, so portions, batches, pages, state
slots and decode steps are all compared against the same numbers.  Weights are a dict of float arrays under the checkpoint's tensor names."""
from __future__ import annotations

import math

import numpy as np

UNIT_EPS = 1e-6   # of the delta rule's unit vectors


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def gelu(z):
    """The tanh form."""
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def unit_rms(x, eps):
    """x over its root mean square along the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    return unit_rms(x, eps) * w


# ------------------------------------------------------------------ around the sublayers
def embed(w, ids):
    return w["embed"][np.asarray(ids)] + w["pos"][:len(ids)]


def norm_of_sum(x, y, w, alpha, eps):
    """What a sublayer's output y makes of the residual x."""
    return rms_norm(alpha * x + y, w, eps)


def side_input(x, ids, w, layer, dim, eps):
    """The token's own vector for this layer, gated by the residual, normed and added to it."""
    p = f"l{layer}.side."
    e = w["side.embed"][np.asarray(ids)][:, layer * dim:(layer + 1) * dim]
    return x + rms_norm((gelu(x @ w[p + "gate"].T) * e) @ w[p + "proj"].T, w[p + "norm"], eps)


def softcap(z, cap):
    return cap * np.tanh(z / cap)


# ------------------------------------------------------------------ gated delta rule
def causal_conv(x, w):
    """x [n, channels] through a causal filter over time per channel: tap j of w [channels, taps] reads taps - 1 - j tokens back."""
    taps, out = w.shape[1], np.zeros_like(x)
    for back in range(taps):
        shifted = np.zeros_like(x)
        shifted[back:] = x[:max(len(x) - back, 0)]
        out += shifted * w[:, taps - 1 - back]
    return out


def unit_vectors(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + UNIT_EPS)


def gated_delta_recurrence(q, k, v, g, beta, state=None):
    """q, k [n, heads, dim], v [n, heads, vdim], decays g and step sizes beta [n, heads].  Returns o [n, heads, vdim] and the state [heads, dim, vdim]."""
    S = np.zeros((q.shape[1], q.shape[2], v.shape[2])) if state is None else state.copy()
    o = np.empty_like(v)
    for t in range(len(q)):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - np.einsum("hde,hd->he", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        o[t] = np.einsum("hde,hd->he", S, q[t])
    return o, S


def delta_decay(a, a_log, dt_bias):
    return np.exp(-np.exp(a_log) * softplus(a + dt_bias))


def delta(h, w, p, mx, eps):
    n, H, G, D, V = len(h), mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q, k, v = (silu(causal_conv(h @ w[p + x].T, w[p + x + ".conv"])) for x in "qkv")
    q, k, v = q.reshape(n, G, D), k.reshape(n, G, D), v.reshape(n, H, V)
    of = np.arange(H) // (H // G)
    q, k = unit_vectors(q)[:, of] * D ** -0.5, unit_vectors(k)[:, of]
    o, _ = gated_delta_recurrence(q, k, v, delta_decay(h @ w[p + "a"].T, w[p + "A_log"], w[p + "dt_bias"]), sigmoid(h @ w[p + "b"].T))
    return ((unit_rms(o, eps) * w[p + "norm"]).reshape(n, H * V) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


# ------------------------------------------------------------------ attention whose values are its keys
def distance_bucket(n, buckets, far):
    """Row of the distance table: one per distance for the first half, then logarithmically spaced up to `far`."""
    half = buckets // 2
    if n < half:
        return n
    return min(buckets - 1, half + math.floor(math.log(n / half) / math.log(far / half) * (buckets - half)))


def visible(n, chunk):
    """[query, key]: the past inside the query's own chunk."""
    i = np.arange(n)
    mask = i[None, :] <= i[:, None]
    return mask if chunk is None else mask & (i[None, :] // chunk == i[:, None] // chunk)


def sink_softmax(s, mask, sink):
    """exp(s) / (exp(sink) + sum exp(s)) over the masked-in entries."""
    s = np.where(mask, s, -np.inf)
    m = np.maximum(s.max(axis=-1, keepdims=True), sink)
    p = np.exp(s - m)
    return p / (np.exp(sink - m) + p.sum(axis=-1, keepdims=True))


def project_keys(h, w, p, mx, eps):
    """(keys, values) [n, kv heads, dim]: the values are the keys in front of their norm."""
    raw = h @ w[p + "k"].T + w[p + "k.b"]
    shape = (len(h), mx["kv_heads"], mx["dim"])
    return rms_norm(raw, w[p + "k.norm"], eps).reshape(shape), raw.reshape(shape)


def attention(h, w, p, mx, eps):
    n, H, G, D = len(h), mx["heads"], mx["kv_heads"], mx["dim"]
    q = rms_norm(h @ w[p + "q"].T + w[p + "q.b"], w[p + "q.norm"], eps).reshape(n, H, D)
    k, v = project_keys(h, w, p, mx, eps)
    rel = w[p + "rel"]
    bucket = np.array([distance_bucket(i, rel.shape[0], mx["bias_max"]) for i in range(n)])
    back = np.maximum(np.arange(n)[:, None] - np.arange(n)[None, :], 0)
    mask = visible(n, (mx.get("mask") or {}).get("size"))
    out = np.empty((n, H, D))
    for a in range(H):
        s = (q[:, a] @ k[:, a // (H // G)].T) * mx["scale"] + rel[bucket[back], a]
        out[:, a] = sink_softmax(s, mask, w[p + "sink"][a]) @ v[:, a // (H // G)]
    return out.reshape(n, H * D) @ w[p + "o"].T


# ------------------------------------------------------------------ RWKV time mixing
def token_shift(h, mu):
    """Every number mixed with the same number of the previous token (zeros in front of the first)."""
    before = np.concatenate([np.zeros_like(h[:1]), h[:-1]])
    return h + (before - h) * mu


def rwkv_recurrence(r, k, v, decay, u, state=None):
    """r, k, v, decay [n, heads, dim], u [heads, dim].  Returns o [n, heads, dim] and the state [heads, dim (key), dim (value)]."""
    S = np.zeros((r.shape[1], r.shape[2], v.shape[2])) if state is None else state.copy()
    o = np.empty_like(v)
    for t in range(len(r)):
        write = k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hde,hd->he", S + u[:, :, None] * write, r[t])
        S = decay[t][:, :, None] * S + write
    return o, S


def rwkv_decay(x, w, p):
    return np.exp(-np.exp(np.tanh(x @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"]))


def time_mixing(h, w, p, mx, eps):
    n, H, D = len(h), mx["heads"], mx["dim"]
    mix = {s: token_shift(h, w[p + "mu." + s]) for s in "rkvgw"}
    r, k, v = ((mix[s] @ w[p + s].T).reshape(n, H, D) for s in "rkv")
    o, _ = rwkv_recurrence(r, k, v, rwkv_decay(mix["w"], w, p).reshape(n, H, D), w[p + "u"])
    return (unit_rms(o, eps).reshape(n, H * D) * w[p + "norm"] * silu(mix["g"] @ w[p + "g"].T)) @ w[p + "o"].T


def parallel(h, w, p, mx, eps):
    return mx["left_scale"] * attention(h, w, p + "left.", mx["left"], eps) + mx["right_scale"] * time_mixing(h, w, p + "right.", mx["right"], eps)


# ------------------------------------------------------------------ feed-forward
def gated_gelu(h, w, p):
    return (gelu(h @ w[p + "gate"].T + w[p + "gate.b"]) * (h @ w[p + "up"].T + w[p + "up.b"])) @ w[p + "down"].T + w[p + "down.b"]


# ------------------------------------------------------------------ the model
def forward(cfg, w, ids, layers_out=None):
    """Logits [n, vocab] of one sequence; layers_out (a list) receives the residual after every layer."""
    eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
    x = embed(w, ids)
    for i, lay in enumerate(cfg["layers"]):
        p = f"l{i}."
        mixer = {"delta": delta, "parallel": parallel}[lay["type"]]
        x = norm_of_sum(x, mixer(x, w, p + "mix.", lay["mixer"], eps), w[p + "norm1"], alpha, eps)
        if lay.get("mlp") is not None:
            x = norm_of_sum(x, gated_gelu(x, w, p + "mlp."), w[p + "norm2"], alpha, eps)
        x = side_input(x, ids, w, i, cfg["token_side"]["dim"], eps)
        if layers_out is not None:
            layers_out.append(x)
    return softcap(rms_norm(x, w["final.norm"], eps) @ w["head"].T, cfg["logit_softcap"])
