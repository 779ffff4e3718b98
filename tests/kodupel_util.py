"""Small random Kodupel models for the tests: configurations, weights, token sequences without close calls, and the error measure against the oracle."""
import numpy as np
import torch

from oracle import kodupel_oracle as orc
from taduzen_util import as_numpy, err  # noqa: F401


def rot(dims=8, base=5000.0, scaling=(4.0, 64, 16.0, 1.0)):
    return {"dims": dims, "base": base, "scaling": None if scaling is None else dict(zip(("factor", "original", "fast", "slow"), scaling))}


def attention(heads=6, kv_heads=2, dim=20, vdim=12, scale=None, kv_from=None, **r):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale, "rot": rot(**r)}
    return ("attention", m if kv_from is None else dict(m, kv_from=kv_from))


def delta(heads=3, dim=24, rank=10):
    return ("general_delta", {"heads": heads, "dim": dim, "_rank": rank})


def moe(ff=20, experts=5, top=2, limit=1.5):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}


def config(layers, width=96, vocab=200, scale=3.0, eps=1e-5):
    return {"architecture": "Kodupel", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps},
            "layers": [{"type": m[0], "mixer": m[1], "mlp": f} for m, f in layers]}


def weights(cfg, seed=0, q_gain=1.0, memory=-2.0, removal=0.0):
    """bf16 tensors of every name the design has.  q_gain sharpens the attention (its queries' norm weight): single keys decide.  memory, removal: means of
    the delta layers' decay and removal biases.  Tokens carry a code of large positive and negative numbers in the columns the routers read, so that scores are
    near 0 or near 1, the corrections decide between equals, and no expert is chosen by a hair (see `sequence`)."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]
    out = {}

    def put(name, *shape, std=None, mean=0.0):
        std = (shape[-1] ** -0.5) if std is None else std
        out[name] = (torch.randn(shape, generator=g) * std + mean).to(torch.bfloat16)

    put("embed", V, W, std=1.0 / cfg["embedding"]["scale"])
    experts = max([lay["mlp"]["router"]["experts"] for lay in cfg["layers"] if lay["mlp"]], default=0)
    coded = min(experts, W)
    code = 2.0 * torch.randint(0, 2, (V, coded), generator=g) - 1.0
    out["embed"][:, :coded] = (14.0 * code / cfg["embedding"]["scale"]).to(torch.bfloat16)
    for i, lay in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", lay["mixer"], lay["mlp"]
        put(p + "norm1", W, std=0.2)
        H, D = m["heads"], m["dim"]
        if lay["type"] == "attention":
            G, U = m["kv_heads"], m["vdim"]
            put(p + "mix.q", H * D, W), put(p + "mix.q.b", H * D, std=0.5), put(p + "mix.q.norm", D, std=0.2 * q_gain, mean=q_gain)
            if m.get("kv_from") is None:
                put(p + "mix.k", G * D, W), put(p + "mix.k.b", G * D, std=0.5), put(p + "mix.k.norm", D, std=0.2, mean=1.0)
                put(p + "mix.v", G * U, W), put(p + "mix.v.b", G * U, std=0.5)
            put(p + "mix.g", H, W), put(p + "mix.o", W, H * U), put(p + "mix.o.b", W, std=0.3)
        else:
            R = m["_rank"]
            for n in "rkvga":
                put(p + f"mix.{n}", H * D, W)
            # (a token's receptance leans on its own key: where the two are orthogonal, a sequence's first outputs are almost nothing, and their direction
            # after the head's norm is decided by rounding)
            out[p + "mix.r"] = (out[p + "mix.r"].float() * 0.6 + out[p + "mix.k"].float() * 0.8).to(torch.bfloat16)
            put(p + "mix.a.b", H * D, std=1.0, mean=removal), put(p + "mix.w0", H * D, std=1.5, mean=memory)
            put(p + "mix.w1", R, W), put(p + "mix.w2", H * D, R, std=2 * R ** -0.5), put(p + "mix.norm", H * D, std=0.2, mean=1.0), put(p + "mix.o", W, H * D)
        if f is None:
            continue
        put(p + "norm2", W, std=0.2)
        E, F = f["router"]["experts"], f["expert"]["ff"]
        router = torch.zeros(E, W)
        cols = torch.randperm(coded, generator=g)[:E] if E <= coded else torch.arange(E) % coded
        router[torch.arange(E), cols] = 0.5
        router += 0.01 * torch.randn(E, W, generator=g)
        out[p + "mlp.router"] = router.to(torch.bfloat16)
        out[p + "mlp.correction"] = ((torch.randperm(E, generator=g) - (E - 1) / 2) * 0.4 / E).to(torch.bfloat16)
        for e in range(E):
            put(f"{p}mlp.e{e}.gate", F, W), put(f"{p}mlp.e{e}.up", F, W), put(f"{p}mlp.e{e}.down", W, F)
    put("final.norm", W, std=0.2)
    put("head", V, W)
    return out


def sequence(cfg, wn, n, seed=1, lead=0.005, layers_out=None, accept=None):
    """(ids, the oracle's logits) of n random tokens in which no expert is chosen by less than `lead` (other tokens are drawn until that holds)."""
    for attempt in range(60):
        ids = np.random.default_rng([seed, attempt]).integers(0, cfg["vocab"], n).astype(np.int32)
        if accept is not None:
            ids = accept(ids)
        leads, outs = [], []
        want = orc.forward(cfg, wn, ids, outs, leads)
        if not leads or min(float(x.min()) for x in leads) >= lead:
            if layers_out is not None:
                layers_out += outs
            return ids, want
    raise AssertionError("every sequence has a close call")


def tokens(cfg, n, seed=1):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).astype(np.int32)


MIXED = [(attention(heads=6, kv_heads=2, dim=20, vdim=12), moe()), (delta(heads=3, dim=24, rank=10), moe(ff=13, experts=4, top=1, limit=0.7)),
         (attention(heads=2, kv_heads=2, dim=40, vdim=24, dims=40, base=300.0, scaling=None), None), (attention(kv_from=0), moe(experts=3, top=3)),
         (delta(heads=2, dim=9, rank=3), None), (attention(heads=2, kv_heads=2, dim=40, vdim=24, dims=40, base=300.0, scaling=None, kv_from=2, scale=0.3), moe(experts=6, top=2))]
CONFIGS = {
    "attention_only": config([(attention(), None)]),
    "one_head": config([(attention(heads=1, kv_heads=1, dim=16, vdim=16, dims=16), None)], width=40),
    "all_heads_share": config([(attention(heads=5, kv_heads=1, dim=8, vdim=40, dims=2, scaling=None), None)]),
    "shared_keys": config([(attention(), None), (attention(kv_from=0, scale=0.4), None), (attention(kv_from=0), None)]),
    "delta_only": config([(delta(), None)]),
    "experts": config([(attention(heads=1, kv_heads=1), moe(ff=30, experts=7, top=3))], width=88, vocab=333),
    "mixed": config(MIXED, width=112, vocab=251, scale=0.7),
    "odd_sizes": config([(attention(heads=3, kv_heads=3, dim=9, vdim=5, dims=6), moe(ff=3, experts=1, top=1)), (delta(heads=1, dim=15, rank=1), moe(ff=5, experts=2, top=1)),
                         (delta(heads=5, dim=13, rank=13), None)], width=21, vocab=53, scale=2.5, eps=1e-3),
    "many_heads": config([(attention(heads=72, kv_heads=2, dim=8, vdim=8, dims=4), None), (delta(heads=40, dim=8, rank=64), None)], width=128),
}
