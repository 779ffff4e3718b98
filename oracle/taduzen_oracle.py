"""Plain restatement of the Taduzen design on the CPU: slow, one function per mechanism, no code shared with the product.

Everything is float64 numpy unless the caller hands in another dtype, whole sequences at once, no cache: the forward pass of one
sequence is a function of its token ids alone, so prompt portions, batches, pages and decode steps are all compared against the same numbers.
Weights are a dict of float arrays under the checkpoint's tensor names (expert tables as integers)."""
from __future__ import annotations

import numpy as np


def dyn_tanh(x, alpha, w, b):
    """Dynamic Tanh: w * tanh(alpha x) + b, element by element; no statistic of x is taken."""
    return np.tanh(alpha * x) * w + b


def rms(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def silu(z):
    return z / (1.0 + np.exp(-z))


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def relu2(z):
    return np.square(np.maximum(z, 0.0))


def visible(n, window):
    """[n, n] bool: query i sees key j.  window: i - j in [0, window); None: every j <= i."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    m = j <= i
    return m if window is None else m & (i - j < window)


def softmax_rows(s, mask):
    s = np.where(mask, s, -np.inf)
    p = np.exp(s - s.max(axis=-1, keepdims=True))
    return p / p.sum(axis=-1, keepdims=True)


def latent_attention(h, w, p, heads, dim, vdim, scale, window, eps):
    """h [n, width] -> [n, width].  p: the mixer's tensor prefix.  Keys and values are spelled out per head (nothing absorbed)."""
    n = h.shape[0]
    q = (h @ w[p + "q"].T).reshape(n, heads, dim)
    c = rms(h @ w[p + "dkv"].T, w[p + "dkv.norm"], eps)
    k = (c @ w[p + "uk"].T).reshape(n, heads, dim)
    v = (c @ w[p + "uv"].T).reshape(n, heads, vdim)
    m = visible(n, window)
    out = np.empty((n, heads, vdim), dtype=h.dtype)
    for a in range(heads):
        out[:, a] = softmax_rows((q[:, a] @ k[:, a].T) * scale, m) @ v[:, a]
    return out.reshape(n, heads * vdim) @ w[p + "o"].T


def dense_ff(h, w, p):
    return relu2(h @ w[p + "up"].T) @ w[p + "down"].T


def gated_expert(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def table_moe(h, ids, w, p, top, shared):
    """Experts by token id: row ids[i] of the table names token i's experts, each with weight 1 / top; plus the gated shared expert."""
    y = np.zeros_like(h)
    for i, t in enumerate(ids):
        for e in w[p + "table"][t][:top]:
            y[i] += gated_expert(h[i:i + 1], w, f"{p}e{int(e)}.")[0] / top
    if shared:
        y += gated_expert(h, w, p + "shared.") * sigmoid(h @ w[p + "shared.sg"].T)
    return y


def forward(cfg, w, ids, layers_out=None):
    """Logits [n, vocab] of one sequence; layers_out (a list) receives the residual stream after every layer."""
    ids = np.asarray(ids)
    eps = cfg["norm"]["eps"]

    def norm(x, name):
        return dyn_tanh(x, w[name + ".alpha"], w[name], w[name + ".b"])

    x = w["embed"][ids]
    for i, lay in enumerate(cfg["layers"]):
        p, mx, ff = f"l{i}.", lay["mixer"], lay.get("mlp")
        mask = mx.get("mask") or {}
        y = latent_attention(norm(x, p + "norm1"), w, p + "mix.", mx["heads"], mx["dim"], mx["vdim"], mx["scale"], mask.get("size"), eps)
        x = x + norm(y, p + "norm1b")
        if ff is not None:
            h = norm(x, p + "norm2")
            if ff["kind"] == "dense":
                y = dense_ff(h, w, p + "mlp.")
            else:
                y = table_moe(h, ids, w, p + "mlp.", ff["router"]["top"], ff.get("shared"))
            x = x + norm(y, p + "norm2b")
        if layers_out is not None:
            layers_out.append(x.copy())
    return (norm(x, "final.norm") @ w["head"].T) * cfg["logit_scale"]
