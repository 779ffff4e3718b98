"""Small random Bezutar models for the tests: configurations, weights, token sequences, and the error measure against the oracle."""
import numpy as np
import torch

from oracle import bezutar_oracle as orc
from taduzen_util import as_numpy, err, tokens  # noqa: F401


def rot(dims, base=5000.0, scaling=(4.0, 64, 16.0, 1.0)):
    return {"dims": dims, "base": base, "scaling": None if scaling is None else dict(zip(("factor", "original", "fast", "slow"), scaling))}


def latent(heads=4, dim=20, rot_dim=8, vdim=12, kv_rank=40, q_rank=24, scale=None, kv_from=None, rot_dims=None, **r):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "scale": (dim + rot_dim) ** -0.5 if scale is None else scale,
         "rot": rot(rot_dim if rot_dims is None else rot_dims, **r)}
    return ("latent_attention", m if kv_from is None else dict(m, kv_from=kv_from))


def mlstm(heads=3, dim=24, vdim=20, gate_cap=9.0):
    return ("mlstm", {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap})


def mingru(width=72):
    return ("mingru", {"width": width})


def dense(ff=80):
    return {"kind": "dense", "ff": ff}


def config(layers, width=96, vocab=200, streams=2, taps=3, eps=1e-5, positions=600, bigram=(61, 7, 3)):
    return {"architecture": "Bezutar", "vocab": vocab, "width": width, "streams": streams, "max_positions": positions, "canon": {"taps": taps}, "norm": {"eps": eps},
            "embedding": {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}, "layers": [{"type": m[0], "mixer": m[1], "mlp": f} for m, f in layers]}


def weights(cfg, seed=0, q_gain=1.0, memory=3.0, entry=0.0, update=-2.0):
    """bf16 tensors of every name the design has.  q_gain sharpens the attention: single keys decide.  memory, entry: means of the mLSTM layers' forget and input gate
    biases; update: of the minGRU layers' update gate bias."""
    g = torch.Generator().manual_seed(seed)
    W, V, S = cfg["width"], cfg["vocab"], cfg["streams"]
    out = {}

    def put(name, *shape, std=None, mean=0.0):
        std = (shape[-1] ** -0.5) if std is None else std
        out[name] = (torch.randn(shape, generator=g) * std + mean).to(torch.bfloat16)

    put("embed", V, W, std=1.0), put("bigram", cfg["embedding"]["bigram"]["buckets"] + 1, W, std=0.6), put("pos", cfg["max_positions"], W, std=0.4)
    for i, lay in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", lay["mixer"], lay["mlp"]
        put(p + "norm1", W, std=0.2), put(p + "canon1", W, cfg["canon"]["taps"], std=0.3)
        for q in ("hc1.", "hc2.") if f else ("hc1.",):
            put(p + q + "in", S, std=0.2, mean=S ** -0.5), put(p + q + "out", S, std=0.3, mean=1.0), put(p + q + "mix", S, S, std=0.2 * S ** -0.5)
            out[p + q + "mix"] += 0.9 * torch.eye(S, dtype=torch.bfloat16)
        if lay["type"] == "latent_attention":
            H, D, T, U, R, Q = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"]
            put(p + "mix.dq", Q, W), put(p + "mix.dq.norm", Q, std=0.2, mean=1.0), put(p + "mix.uq", H * (D + T), Q, std=q_gain * Q ** -0.5)
            if m.get("kv_from") is None:
                put(p + "mix.dkv", R + T, W), put(p + "mix.dkv.norm", R, std=0.2, mean=1.0)
            put(p + "mix.uk", H * D, R), put(p + "mix.uv", H * U, R), put(p + "mix.sink", H, std=1.5), put(p + "mix.g", H, W), put(p + "mix.o", W, H * U)
        elif lay["type"] == "mlstm":
            H, D, U = m["heads"], m["dim"], m["vdim"]
            put(p + "mix.q", H * D, W), put(p + "mix.k", H * D, W), put(p + "mix.v", H * U, W), put(p + "mix.g", H * U, W), put(p + "mix.o", W, H * U)
            # (a token's query leans on its own key: where the two are orthogonal, a sequence's first outputs are almost nothing, and their direction after the head's
            # norm is decided by rounding)
            out[p + "mix.q"] = (out[p + "mix.q"].float() * 0.4 + out[p + "mix.k"].float() * 0.92).to(torch.bfloat16)
            put(p + "mix.norm", H * U, std=0.2, mean=1.0), put(p + "mix.i", H, W), put(p + "mix.i.b", H, std=0.5, mean=entry), put(p + "mix.f", H, W), put(p + "mix.f.b", H, std=1.0, mean=memory)
        else:
            N = m["width"]
            put(p + "mix.z", N, W), put(p + "mix.z.b", N, std=1.0, mean=update), put(p + "mix.x", N, W), put(p + "mix.x.b", N, std=0.5), put(p + "mix.g", N, W), put(p + "mix.o", W, N)
        if f is not None:
            put(p + "norm2", W, std=0.2), put(p + "mlp.up", f["ff"], W), put(p + "mlp.down", W, f["ff"]), put(p + "mlp.act", 2, std=0.7)
    put("final.norm", W, std=0.2)
    put("head", V, W)
    return out


def sequence(cfg, wn, n, seed=1):
    ids = tokens(cfg, n, seed)
    return ids, orc.forward(cfg, wn, ids)


def plain(w, cfg):
    """Takes away what stands between the token's vector and the mixers: streams that add up, no convolution, no bigrams, no positions."""
    for n, t in w.items():
        if n in ("bigram", "pos") or "canon1" in n:
            t.zero_()
        elif ".hc" in n:
            t.copy_(torch.eye(cfg["streams"]) if n.endswith("mix") else torch.ones(cfg["streams"]) / (cfg["streams"] if n.endswith("in") else 1))
    return w


MIXED = [(latent(), dense()), (mingru(), dense(33)), (mlstm(), dense(72)), (latent(heads=3, dim=12, rot_dim=8, vdim=28, kv_rank=40, q_rank=50, kv_from=0, scale=0.3), None),
         (mlstm(heads=2, dim=9, vdim=7, gate_cap=4.0), None), (latent(heads=2, dim=33, rot_dim=16, vdim=16, kv_rank=20, q_rank=16, base=300.0, scaling=None), dense(24)),
         (mingru(50), None), (latent(heads=5, dim=8, rot_dim=16, vdim=8, kv_rank=20, q_rank=8, kv_from=5, base=300.0, scaling=None), dense(40))]
CONFIGS = {
    "attention_only": config([(latent(), None)]),
    "one_head": config([(latent(heads=1, dim=16, rot_dim=2, vdim=16, kv_rank=16, q_rank=16, scaling=None), None)], width=40, streams=1, taps=1),
    "shared_latents": config([(latent(), None), (latent(kv_from=0, scale=0.4), dense()), (latent(kv_from=0, heads=7), None)], taps=2),
    "mlstm_only": config([(mlstm(), None)], taps=4),
    "mingru_only": config([(mingru(), None)], streams=4),
    "dense_only": config([(mingru(8), dense(200))], width=88, vocab=333),
    "mixed": config(MIXED, width=112, vocab=251, streams=3, taps=5, bigram=(97, 31, 5)),
    "odd_sizes": config([(latent(heads=3, dim=9, rot_dim=6, vdim=5, kv_rank=7, q_rank=5), dense(3)), (mlstm(heads=1, dim=15, vdim=9), dense(13)), (mingru(13), None),
                         (mlstm(heads=5, dim=13, vdim=19), None)], width=21, vocab=53, streams=5, taps=7, eps=1e-3, bigram=(1, 5, 9)),
    "many_heads": config([(latent(heads=72, dim=8, rot_dim=4, vdim=8), None), (mlstm(heads=40, dim=8, vdim=8), None)], width=128, streams=2),
}
