"""Kodupel: softmax attention (grouped heads, query / key / value norms, partial interleaved rotation with YaRN scaling, a denominator sink, per-head output
gates, keys and values shared between layers) and generalised delta-rule layers, in any order; RMS norms behind the sublayers only; mixtures of clipped
gated experts behind a sigmoid router.

config.json lists the layers one by one ("layers"), each with its own sizes; tensors are named l<i>.* (norm1, norm2, mix.*, mlp.*), embed, final.norm, head.
The arithmetic runs in the native layer stack (models/layer_stack.py); this file reads the configuration and packs the weights."""
from __future__ import annotations

import math

import torch

from .. import base
from ... import _ffi
from ..layer_stack import LayerStackModel, Norm, interleave, pack_linear, pad, pad_head_columns, pad_head_rows, up8, yarn_frequencies

EXPERT_SLOPE = 1.702          # of the experts' sigmoid
DECAY_SCALE = math.exp(-0.5)  # a delta layer's log decay lies in (-DECAY_SCALE, 0)
UNIT_KEY_EPS = 1e-6
SINK = 1.0                    # what the softmax's denominator has besides the keys


class ScalingArgs(base.BaseModelArgs):
    factor: float
    original: float
    fast: float
    slow: float


class RotArgs(base.BaseModelArgs):
    dims: int
    base: float
    scaling: ScalingArgs | None = None


class MixerArgs(base.BaseModelArgs):
    heads: int
    dim: int
    kv_heads: int = 0          # attention, from here on
    vdim: int = 0
    scale: float = 0.0
    rot: RotArgs | None = None
    kv_from: int | None = None


class ExpertArgs(base.BaseModelArgs):
    ff: int
    limit: float


class RouterArgs(base.BaseModelArgs):
    experts: int
    top: int


class MlpArgs(base.BaseModelArgs):
    kind: str
    expert: ExpertArgs
    router: RouterArgs


class LayerArgs(base.BaseModelArgs):
    type: str
    mixer: MixerArgs
    mlp: MlpArgs | None = None


class NormArgs(base.BaseModelArgs):
    eps: float


class EmbeddingArgs(base.BaseModelArgs):
    scale: float


class ModelArgs(base.BaseModelArgs):
    architecture: str = "Kodupel"
    layers: list[LayerArgs]
    vocab: int
    width: int
    embedding: EmbeddingArgs
    norm: NormArgs


class Model(LayerStackModel):
    model_type = "kodupel"

    def __init__(self, args: ModelArgs, weights: dict[str, torch.Tensor], dtype: torch.dtype = torch.bfloat16):
        """weights: the checkpoint's tensors on the device (bf16).  dtype: bfloat16, or float32 for 32-bit arithmetic throughout."""
        W, eps = args.width, args.norm.eps

        def get(name: str, *shape: int) -> torch.Tensor:
            t = weights.get(name)
            if t is None:
                raise ValueError(f"{name} is missing from the checkpoint")
            if tuple(t.shape) != shape:
                raise ValueError(f"{name}: expected {list(shape)}, got {list(t.shape)}")
            return t

        def norm(name: str) -> Norm:  # (stored as the difference from one)
            return Norm(_ffi.PIE_NORM_RMS, eps, pad(1.0 + get(name, W).float()[None], 1, up8(W))[0])

        def pack(w: torch.Tensor) -> torch.Tensor:
            return pack_linear(w, dtype)

        def flat(name: str, *shape: int) -> torch.Tensor:
            return get(name, *shape).float().contiguous()

        def attention(p: str, m: MixerArgs) -> dict:
            H, G, D, V = m.heads, m.kv_heads, m.dim, m.vdim
            own = m.kv_from is None
            if G < 1 or H % G:
                raise ValueError(f"{p}: {H} heads over {G} key/value heads")
            rows = [pad_head_rows(get(p + "q", H * D, W), H, D)]
            bias = [pad_head_rows(get(p + "q.b", H * D)[:, None], H, D)]
            if own:
                rows += [pad_head_rows(get(p + "k", G * D, W), G, D), pad_head_rows(get(p + "v", G * V, W), G, V)]
                bias += [pad_head_rows(get(p + "k.b", G * D)[:, None], G, D), pad_head_rows(get(p + "v.b", G * V)[:, None], G, V)]
            rows.append(pad(get(p + "g", H, W), up8(H), W))
            bias.append(torch.zeros(up8(H), 1, dtype=torch.bfloat16, device=rows[0].device))
            out = {"mixer": _ffi.PIE_MIXER_ATTENTION, "heads": H, "dim": D, "vdim": V, "kv_heads": G, "kv_from": -1 if own else m.kv_from, "scale": m.scale,
                   "value_norm": 1, "out_gate": 1, "out_scale": 1.0, "sink": SINK, "w_in": pack(torch.cat(rows)), "in_bias": torch.cat(bias)[:, 0].to(torch.bfloat16).contiguous(),
                   "q_norm": flat(p + "q.norm", D), "w_o": pack(pad_head_columns(get(p + "o", W, H * V), H, V)),
                   "o_bias": get(p + "o.b", W).to(torch.bfloat16).contiguous()}
            if own:
                out["k_norm"] = flat(p + "k.norm", D)
            if m.rot is not None and m.rot.dims > 0:
                s = m.rot.scaling
                freq, gain = yarn_frequencies(m.rot.dims, m.rot.base, None if s is None else (s.factor, s.original, s.fast, s.slow))
                out |= {"rot_dims": m.rot.dims, "rot_gain": gain, "rot_freq": freq.to(rows[0].device)}
            return out

        def delta(p: str, m: MixerArgs) -> dict:
            H, D = m.heads, m.dim
            n = H * D
            R = weights[p + "w1"].shape[0] if p + "w1" in weights else 0  # (the decay's rank stands in the tensors only)
            rows = [pad_head_rows(get(p + x, n, W), H, D) for x in ("r", "k", "v", "g", "a")] + [pad(get(p + "w1", R, W), up8(R), W)]
            bias = torch.zeros(sum(r.shape[0] for r in rows), dtype=torch.bfloat16, device=rows[0].device)
            at = 4 * rows[0].shape[0]
            bias[at:at + rows[4].shape[0]] = pad_head_rows(get(p + "a.b", n)[:, None], H, D)[:, 0]
            return {"mixer": _ffi.PIE_MIXER_DELTA, "heads": H, "dim": D, "rank": R, "kv_from": -1, "decay_scale": DECAY_SCALE, "unit_eps": UNIT_KEY_EPS,
                    "w_in": pack(torch.cat(rows)), "in_bias": bias, "w_decay": pad(get(p + "w2", n, R).to(torch.bfloat16), n, up8(R)), "decay_bias": flat(p + "w0", n),
                    "o_norm": flat(p + "norm", n), "w_o": pack(pad_head_columns(get(p + "o", W, n), H, D))}

        def mixture(p: str, ff: MlpArgs) -> dict:
            E, F = ff.router.experts, ff.expert.ff
            F8 = up8(F)  # (padded with zero rows and columns: the activation of a zero gate is zero)

            def gated(q: str):
                return (pack(interleave(pad(get(q + "gate", F, W), F8, W), pad(get(q + "up", F, W), F8, W))), pack(pad(get(q + "down", W, F), W, F8)))
            experts = [gated(f"{p}e{e}.") for e in range(E)]
            return {"ff": _ffi.PIE_FF_ROUTED_MOE, "ff_size": F8, "experts": E, "top": ff.router.top, "act": _ffi.PIE_ACT_CLIPPED, "act_alpha": EXPERT_SLOPE,
                    "act_limit": ff.expert.limit, "w_router": pack(get(p + "router", E, W)), "w_router_rows": pad(get(p + "router", E, W).to(torch.bfloat16), E, up8(W)),
                    "correction": flat(p + "correction", E),
                    "w_gate_up": torch.cat([e[0] for e in experts]), "w_expert_down": torch.cat([e[1] for e in experts])}

        if not args.layers:
            raise ValueError("a model has at least one layer")
        mixers = {"attention": attention, "general_delta": delta}
        layers = []
        for i, lay in enumerate(args.layers):
            p = f"l{i}."
            if lay.type not in mixers:
                raise ValueError(f"layer {i}: unknown mixer {lay.type!r}")
            fields = {"post1": norm(p + "norm1"), "eps": eps} | mixers[lay.type](p + "mix.", lay.mixer)
            if lay.mlp is not None:
                if lay.mlp.kind != "moe":
                    raise ValueError(f"layer {i}: unknown feed-forward {lay.mlp.kind!r}")
                fields |= {"post2": norm(p + "norm2")} | mixture(p + "mlp.", lay.mlp)
            layers.append(fields)
        super().__init__(args, dtype, W, args.vocab, 1.0, layers, get("embed", args.vocab, W).to(torch.bfloat16).contiguous(), pack(get("head", args.vocab, W)),
                         norm("final.norm"), embed_scale=args.embedding.scale)
