"""Small random Taduzen models for the tests: configurations, weights, and the error measure against the oracle."""
import numpy as np
import torch


def latent(heads=4, dim=16, vdim=16, rank=48, window=40, scale=None):
    return {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "scale": dim ** -0.5 if scale is None else scale,
            "mask": None if window is None else {"size": window}}


def dense(ff=80):
    return {"kind": "dense", "ff": ff}


def moe(ff=24, experts=5, top=2, shared=40):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}, "shared": None if shared is None else {"ff": shared}}


def config(layers, width=96, vocab=200, logit_scale=1.5, eps=1e-5):
    return {"architecture": "Taduzen", "vocab": vocab, "width": width, "logit_scale": logit_scale, "norm": {"eps": eps},
            "layers": [{"type": "latent_attention", "mixer": m, "mlp": f} for m, f in layers]}


def weights(cfg, seed=0, q_gain=1.0):
    """bf16 (int32 tables) tensors of every name the design has.  q_gain sharpens the attention: single keys decide."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]
    out = {}

    def put(name, *shape, std=None, mean=0.0):
        std = (shape[-1] ** -0.5) if std is None else std
        out[name] = (torch.randn(shape, generator=g) * std + mean).to(torch.bfloat16)

    def norm(name):
        put(name, W, std=0.2, mean=1.0)
        put(name + ".b", W, std=0.2)
        out[name + ".alpha"] = (0.4 + torch.rand((), generator=g)).to(torch.bfloat16)

    put("embed", V, W, std=1.0)
    for i, lay in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", lay["mixer"], lay["mlp"]
        norm(p + "norm1"), norm(p + "norm1b")
        put(p + "mix.q", m["heads"] * m["dim"], W, std=q_gain * W ** -0.5)
        put(p + "mix.dkv", m["kv_rank"], W)
        put(p + "mix.dkv.norm", m["kv_rank"], std=0.2, mean=1.0)
        put(p + "mix.uk", m["heads"] * m["dim"], m["kv_rank"])
        put(p + "mix.uv", m["heads"] * m["vdim"], m["kv_rank"])
        put(p + "mix.o", W, m["heads"] * m["vdim"])
        if f is None:
            continue
        norm(p + "norm2"), norm(p + "norm2b")
        if f["kind"] == "dense":
            put(p + "mlp.up", f["ff"], W), put(p + "mlp.down", W, f["ff"])
            continue
        E, top = f["router"]["experts"], f["router"]["top"]
        out[p + "mlp.table"] = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(V)]).to(torch.int32)
        for e in [f"e{e}" for e in range(E)] + (["shared"] if f["shared"] else []):
            F = f["shared"]["ff"] if e == "shared" else f["expert"]["ff"]
            put(f"{p}mlp.{e}.gate", F, W, std=2 * W ** -0.5), put(f"{p}mlp.{e}.up", F, W), put(f"{p}mlp.{e}.down", W, F, std=2 * F ** -0.5)
        if f["shared"]:
            put(p + "mlp.shared.sg", 1, W)
    norm("final.norm")
    put("head", V, W)
    return out


def as_numpy(w):
    return {k: v.numpy() if v.dtype == torch.int32 else v.double().numpy() for k, v in w.items()}


def err(got, want):
    """Worst row: rms of the difference (row means taken off) over the rms of the expected rows."""
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want, dtype=np.float64)
    d, c = got - want, want - want.mean(-1, keepdims=True)
    d = d - d.mean(-1, keepdims=True)
    return float(np.sqrt((d * d).mean(-1)).max() / np.sqrt((c * c).mean()))


def tokens(cfg, n, seed=1):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).astype(np.int32)
