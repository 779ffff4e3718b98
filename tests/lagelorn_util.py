"""Small random Lagelorn models for the tests: configurations, weights, token sequences, and the error measure against the oracle."""
import torch

from oracle import lagelorn_oracle as orc
from taduzen_util import as_numpy, err, tokens  # noqa: F401


def delta(heads=3, kv_heads=None, dim=20, vdim=28, conv=3):
    return ("delta", {"heads": heads, "kv_heads": kv_heads or heads, "dim": dim, "vdim": vdim, "conv": conv})


def left(heads=4, kv_heads=2, dim=24, scale=None, bias_max=90, chunk=70):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5 if scale is None else scale, "bias_max": bias_max, "mask": chunk and {"size": chunk}}


def right(heads=3, dim=20):
    return {"heads": heads, "dim": dim}


def parallel(a=None, b=None, scales=(0.8, 1.3)):
    return ("parallel", {"left": a or left(), "right": b or right(), "left_scale": scales[0], "right_scale": scales[1]})


def dense(ff=80):
    return {"kind": "dense", "ff": ff}


def config(layers, width=96, vocab=200, side=16, eps=1e-5, alpha=1.7, cap=4.0, positions=640):
    return {"architecture": "Lagelorn", "vocab": vocab, "width": width, "max_positions": positions, "token_side": {"dim": side}, "norm": {"eps": eps}, "postln_alpha": alpha,
            "logit_softcap": cap, "layers": [{"type": m[0], "mixer": m[1], "mlp": f} for m, f in layers]}


def weights(cfg, seed=0, q_gain=1.0, rel_rows=12, rank=10, decay=-3.0, spread=1.5, sink=0.0):
    """bf16 tensors of every name the design has.  q_gain sharpens the attention: single keys decide.  decay, spread: mean and deviation of what decays are made of (w0, dt_bias): large means
    states that forget fast; sink: mean of the sinks."""
    g = torch.Generator().manual_seed(seed)
    W, V, S = cfg["width"], cfg["vocab"], cfg["token_side"]["dim"]
    out = {}

    def put(name, *shape, std=None, mean=0.0):
        std = (shape[-1] ** -0.5) if std is None else std
        out[name] = (torch.randn(shape, generator=g) * std + mean).to(torch.bfloat16)

    def lean(a, b):
        """(a token's query leans on its own key: where the two are orthogonal, a sequence's first outputs are almost nothing, and their direction after the head's norm is decided by rounding)"""
        out[a] = (out[a].float() * 0.4 + out[b].float() * 0.92).to(torch.bfloat16)

    put("embed", V, W, std=1.0), put("pos", cfg["max_positions"], W, std=0.4), put("side.embed", V, len(cfg["layers"]) * S, std=1.0)
    for i, lay in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", lay["mixer"], lay["mlp"]
        put(p + "norm1", W, std=0.2, mean=1.0)
        put(p + "side.gate", S, W), put(p + "side.proj", W, S), put(p + "side.norm", W, std=0.2, mean=0.5)
        if lay["type"] == "delta":
            H, G, D, U, T = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
            for n, c in (("q", G * D), ("k", G * D), ("v", H * U)):
                put(p + f"mix.{n}", c, W), put(p + f"mix.{n}.conv", c, T, std=0.4)
                out[p + f"mix.{n}.conv"][:, -1] += 0.8
            lean(p + "mix.q", p + "mix.k"), lean(p + "mix.q.conv", p + "mix.k.conv")
            put(p + "mix.g", H * U, W), put(p + "mix.b", H, W), put(p + "mix.a", H, W), put(p + "mix.A_log", H, std=0.7), put(p + "mix.dt_bias", H, std=spread, mean=decay)
            put(p + "mix.norm", U, std=0.2, mean=1.0), put(p + "mix.o", W, H * U)
        else:
            a, b = m["left"], m["right"]
            H, G, D, q = a["heads"], a["kv_heads"], a["dim"], p + "mix.left."
            put(q + "q", H * D, W, std=q_gain * W ** -0.5), put(q + "q.b", H * D, std=0.3), put(q + "k", G * D, W), put(q + "k.b", G * D, std=0.3)
            put(q + "q.norm", H * D, std=0.2, mean=q_gain), put(q + "k.norm", G * D, std=0.2, mean=1.0)
            put(q + "rel", rel_rows, H, std=1.0), put(q + "sink", H, std=1.0, mean=sink), put(q + "o", W, H * D)
            H, D, q = b["heads"], b["dim"], p + "mix.right."
            for n in "rkvgw":
                put(q + "mu." + n, W, std=0.3, mean=0.5)
            for n in "rkvg":
                put(q + n, H * D, W)
            lean(q + "r", q + "k")
            put(q + "w1", rank, W), put(q + "w2", H * D, rank), put(q + "w0", H * D, std=spread, mean=decay), put(q + "u", H, D, std=0.4, mean=1.0)
            put(q + "norm", H * D, std=0.2, mean=1.0), put(q + "o", W, H * D)
        if f is not None:
            put(p + "norm2", W, std=0.2, mean=1.0)
            for n in ("gate", "up"):
                put(p + f"mlp.{n}", f["ff"], W), put(p + f"mlp.{n}.b", f["ff"], std=0.3)
            put(p + "mlp.down", W, f["ff"]), put(p + "mlp.down.b", W, std=0.3)
    put("final.norm", W, std=0.2, mean=1.0)
    put("head", V, W, std=2.0 * W ** -0.5)
    return out


def sequence(cfg, wn, n, seed=1):
    ids = tokens(cfg, n, seed)
    return ids, orc.forward(cfg, wn, ids)


def only(w, keep):
    """Takes away what stands beside the mechanisms under test: positions and side inputs, and of every parallel layer the side that is not in `keep`."""
    for n, t in w.items():
        if n == "pos" or n.endswith("side.norm") or any(f"mix.{s}.o" in n for s in {"left", "right"} - set(keep)):
            t.zero_()
    return w


MIXED = [(parallel(), dense()), (delta(), None), (delta(heads=4, kv_heads=2, dim=16, vdim=40, conv=5), dense(33)),
         (parallel(left(heads=6, kv_heads=2, dim=9, bias_max=40, chunk=33, scale=0.5), right(heads=2, dim=33), (1.2, 0.5)), None),
         (parallel(left(heads=3, kv_heads=3, dim=40, chunk=None), right(heads=5, dim=7)), dense(24))]
CONFIGS = {
    "delta_only": config([(delta(), None)]),
    "parallel_only": config([(parallel(), None)]),
    "dense_behind_delta": config([(delta(heads=1, dim=8, vdim=8, conv=1), dense(200))], width=88, vocab=333, side=8),
    "one_head": config([(parallel(left(heads=1, kv_heads=1, dim=16), right(heads=1, dim=16)), None)], width=40, side=6, alpha=1.0),
    "mixed": config(MIXED, width=112, vocab=251),
    "odd_sizes": config([(parallel(left(heads=3, kv_heads=1, dim=5, bias_max=17, chunk=9), right(heads=1, dim=13)), dense(13)), (delta(heads=5, kv_heads=1, dim=13, vdim=19, conv=2), None),
                         (delta(heads=3, dim=11, vdim=21, conv=7), dense(3))], width=37, vocab=53, side=21, eps=0.02, alpha=2.3, cap=2.0),
    "many_heads": config([(parallel(left(heads=72, kv_heads=8, dim=8), right(heads=40, dim=8)), None), (delta(heads=40, kv_heads=20, dim=8, vdim=8), None)], width=128),
}
