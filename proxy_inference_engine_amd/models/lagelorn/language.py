"""Lagelorn: gated delta-rule layers, and layers that run an attention and RWKV time mixing side by side on the same input, in any order; RMS norms over the scaled residual plus
a sublayer's output (post-norm), gated gelu feed-forwards, and per layer a vector of the token that the residual gates (side input); learned position vectors, capped logits.
The attention sees its own chunk of positions, adds a learned number by head and distance bucket, has a learned sink per head, norms queries and keys over all heads at once, and
its values are its keys in front of their norm.

config.json lists the layers one by one ("layers"), each with its own sizes; tensors are named l<i>.* (norm1, norm2, mix.*, mlp.*, side.*), embed, pos, side.embed, final.norm, head.
The arithmetic runs in the native layer stack (models/layer_stack.py); this file reads the configuration and packs the weights."""
from __future__ import annotations

import math

import torch

from .. import base
from ... import _ffi
from ..layer_stack import Embedding, LayerStackModel, Norm, interleave, pack_linear, pad, pad_head_columns, pad_head_rows, up8

UNIT_EPS = 1e-6   # of the delta rule's unit queries and keys


class MaskArgs(base.BaseModelArgs):
    size: int


class AttentionArgs(base.BaseModelArgs):
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    bias_max: float
    mask: MaskArgs | None = None


class TimeMixArgs(base.BaseModelArgs):
    heads: int
    dim: int


class MixerArgs(base.BaseModelArgs):
    heads: int = 0             # delta
    kv_heads: int = 0
    dim: int = 0
    vdim: int = 0
    conv: int = 0
    left: AttentionArgs | None = None   # parallel, from here on
    right: TimeMixArgs | None = None
    left_scale: float = 0.0
    right_scale: float = 0.0


class MlpArgs(base.BaseModelArgs):
    kind: str
    ff: int


class LayerArgs(base.BaseModelArgs):
    type: str
    mixer: MixerArgs
    mlp: MlpArgs | None = None


class NormArgs(base.BaseModelArgs):
    eps: float


class SideArgs(base.BaseModelArgs):
    dim: int


class ModelArgs(base.BaseModelArgs):
    architecture: str = "Lagelorn"
    layers: list[LayerArgs]
    vocab: int
    width: int
    max_positions: int
    norm: NormArgs
    postln_alpha: float
    token_side: SideArgs
    logit_softcap: float


def distance_buckets(buckets: int, far: float) -> list[int]:
    """Row of the distance table for every distance from 0 on, up to the first that takes the last row (as all behind it do): one row per distance for the first half of the table,
    then logarithmically spaced up to `far`."""
    half = buckets // 2
    out = list(range(half))
    if half < 1 or far <= half:
        raise ValueError(f"distance buckets: {buckets} rows up to {far}")
    while not out or out[-1] < buckets - 1:
        out.append(min(buckets - 1, half + math.floor(math.log(len(out) / half) / math.log(far / half) * (buckets - half))))
    return out


class Model(LayerStackModel):
    model_type = "lagelorn"

    def __init__(self, args: ModelArgs, weights: dict[str, torch.Tensor], dtype: torch.dtype = torch.bfloat16):
        """weights: the checkpoint's tensors on the device (bf16).  dtype: bfloat16, or float32 for 32-bit arithmetic throughout."""
        W, eps = args.width, args.norm.eps

        def get(name: str, *shape: int) -> torch.Tensor:
            t = weights.get(name)
            if t is None:
                raise ValueError(f"{name} is missing from the checkpoint")
            if len(t.shape) != len(shape) or any(n not in (m, -1) for n, m in zip(shape, t.shape)):  # (-1: the size stands in the tensor only)
                raise ValueError(f"{name}: expected {list(shape)}, got {list(t.shape)}")
            return t

        def norm(name: str) -> Norm:
            return Norm(_ffi.PIE_NORM_RMS, eps, pad(get(name, W).float()[None], 1, up8(W))[0])

        def pack(w: torch.Tensor) -> torch.Tensor:
            return pack_linear(w, dtype)

        def flat(name: str, *shape: int) -> torch.Tensor:
            return get(name, *shape).float().contiguous()

        def bf16(t: torch.Tensor) -> torch.Tensor:
            return t.to(torch.bfloat16).contiguous()

        def heads_vector(name: str, heads: int, n: int) -> torch.Tensor:  # [heads * n] -> [heads * up8(n)]
            return pad_head_rows(get(name, heads * n)[:, None], heads, n)[:, 0]

        def groups(p: str, heads: int, kv_heads: int) -> None:
            if kv_heads < 1 or heads % kv_heads:
                raise ValueError(f"{p}: {heads} heads over {kv_heads} key/value heads")

        def delta(p: str, m: MixerArgs) -> dict:
            H, G, D, V, taps = m.heads, m.kv_heads, m.dim, m.vdim, m.conv
            groups(p, H, G)
            rows = [pad_head_rows(get(p + n, h * d, W), h, d) for n, h, d in (("q", G, D), ("k", G, D), ("v", H, V), ("g", H, V))] + [pad(get(p + n, H, W), up8(H), W) for n in "ba"]
            conv = torch.cat([pad_head_rows(get(p + n + ".conv", h * d, taps).float(), h, d) for n, h, d in (("q", G, D), ("k", G, D), ("v", H, V))]).T.contiguous()
            return {"mixer": _ffi.PIE_MIXER_GATED_DELTA, "heads": H, "kv_heads": G, "dim": D, "vdim": V, "kv_from": -1, "scale": D ** -0.5, "unit_eps": UNIT_EPS, "mix_conv": conv, "mix_taps": taps,
                    "w_in": pack(torch.cat(rows)), "decay_rate": flat(p + "A_log", H).exp(), "decay_bias": flat(p + "dt_bias", H), "o_norm": flat(p + "norm", V),
                    "w_o": pack(pad_head_columns(get(p + "o", W, H * V), H, V))}

        def attention(p: str, m: AttentionArgs) -> dict:
            H, G, D = m.heads, m.kv_heads, m.dim
            groups(p, H, G)
            if m.vdim != D:
                raise ValueError(f"{p}: values are the keys, but have {m.vdim} numbers instead of {D}")
            rel = get(p + "rel", -1, H).float()
            rel = rel[torch.tensor(distance_buckets(rel.shape[0], m.bias_max), device=rel.device)].T.contiguous()  # [H][far + 1]
            return {"mixer": _ffi.PIE_MIXER_ATTENTION, "heads": H, "kv_heads": G, "dim": D, "vdim": D, "kv_from": -1, "scale": m.scale, "row_norm": 1, "chunk": m.mask.size if m.mask else 0,
                    "distance": rel, "far": rel.shape[1] - 1, "head_sink": flat(p + "sink", H), "w_in": pack(torch.cat([pad_head_rows(get(p + "q", H * D, W), H, D), pad_head_rows(get(p + "k", G * D, W), G, D)])),
                    "in_bias": bf16(torch.cat([heads_vector(p + "q.b", H, D), heads_vector(p + "k.b", G, D)])), "q_norm": heads_vector(p + "q.norm", H, D).float().contiguous(),
                    "k_norm": heads_vector(p + "k.norm", G, D).float().contiguous()}

        def time_mixing(p: str, m: TimeMixArgs) -> dict:
            H, D = m.heads, m.dim
            R = get(p + "w1", -1, W).shape[0]  # (the decay's rank stands in the tensors only)
            mu = torch.stack([pad(get(p + "mu." + s, W).float()[None], 1, (W + 63) // 64 * 64)[0] for s in "rkvgw"])
            return {"heads": H, "dim": D, "rank": R, "mu": mu, **{"w_" + n: pack(pad_head_rows(get(p + t, H * D, W), H, D)) for n, t in (("r", "r"), ("k", "k"), ("v", "v"), ("gate", "g"))},
                    "w_low": pack(pad(get(p + "w1", R, W), up8(R), W)), "w_decay": pad(bf16(get(p + "w2", H * D, R)), H * D, up8(R)), "decay_bias": flat(p + "w0", H * D),
                    "bonus": flat(p + "u", H, D).flatten(), "o_norm": flat(p + "norm", H * D)}

        def parallel(p: str, m: MixerArgs) -> dict:
            if m.left is None or m.right is None:
                raise ValueError(f"{p}: a parallel mixer has two sides")
            l, r = m.left, m.right
            out = torch.cat([pad_head_columns(get(p + "left.o", W, l.heads * l.dim), l.heads, l.dim), pad_head_columns(get(p + "right.o", W, r.heads * r.dim), r.heads, r.dim)], dim=1)
            return attention(p + "left.", l) | {"out_scale": m.left_scale, "time_mix": time_mixing(p + "right.", r) | {"out_scale": m.right_scale}, "w_o": pack(out)}

        def dense(p: str, ff: MlpArgs) -> dict:
            F, F8 = ff.ff, up8(ff.ff)  # (padded with zero rows and columns: the gelu of zero is zero)
            bias = interleave(*(pad(get(p + n + ".b", F)[:, None], F8, 1) for n in ("gate", "up")))[:, 0]
            return {"ff": _ffi.PIE_FF_GEGLU, "ff_size": F8, "w_up": pack(interleave(pad(get(p + "gate", F, W), F8, W), pad(get(p + "up", F, W), F8, W))), "up_bias": bf16(bias),
                    "w_down": pack(pad(get(p + "down", W, F), W, F8)), "down_bias": bf16(get(p + "down.b", W))}

        if not args.layers:
            raise ValueError("a model has at least one layer")
        S = args.token_side.dim
        mixers = {"delta": delta, "parallel": parallel}
        layers = []
        for i, lay in enumerate(args.layers):
            p = f"l{i}."
            if lay.type not in mixers:
                raise ValueError(f"layer {i}: unknown mixer {lay.type!r}")
            fields = {"post1": norm(p + "norm1"), "eps": eps, "norm_after": 1, "residual_scale": args.postln_alpha, "w_side_gate": pack(get(p + "side.gate", S, W)),
                      "w_side_proj": pack(get(p + "side.proj", W, S)), "side_norm": norm(p + "side.norm")} | mixers[lay.type](p + "mix.", lay.mixer)
            if lay.mlp is not None:
                if lay.mlp.kind != "dense":
                    raise ValueError(f"layer {i}: unknown feed-forward {lay.mlp.kind!r}")
                fields |= {"post2": norm(p + "norm2")} | dense(p + "mlp.", lay.mlp)
            layers.append(fields)
        super().__init__(args, dtype, W, args.vocab, 1.0, layers, bf16(get("embed", args.vocab, W)), pack(get("head", args.vocab, W)), norm("final.norm"),
                         embedding=Embedding(positions=bf16(get("pos", args.max_positions, W)), side=bf16(get("side.embed", args.vocab, len(layers) * S))), logit_cap=args.logit_softcap)
