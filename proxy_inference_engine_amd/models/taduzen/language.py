"""Taduzen: latent attention without positions under a sliding window, Dynamic Tanh norms in front of and behind every sublayer, and feed-forwards that
are dense (squared relu) or mixtures whose experts a table picks by token id, beside a gated shared expert.

config.json lists the layers one by one ("layers"), each with its own sizes; tensors are named l<i>.* (norm1, norm1b, norm2, norm2b, mix.*, mlp.*),
embed, final.norm, head.  The arithmetic runs in the native layer stack (models/layer_stack.py); this file reads the configuration and packs the weights."""
from __future__ import annotations

import torch

from .. import base
from ... import _ffi
from ..layer_stack import LayerStackModel, Norm, interleave, pack_linear, pad, pad_head_columns, pad_head_rows, up8


class MaskArgs(base.BaseModelArgs):
    size: int


class MixerArgs(base.BaseModelArgs):
    heads: int
    dim: int
    vdim: int
    kv_rank: int
    scale: float
    mask: MaskArgs | None = None


class ExpertArgs(base.BaseModelArgs):
    ff: int


class RouterArgs(base.BaseModelArgs):
    experts: int
    top: int


class MlpArgs(base.BaseModelArgs):
    kind: str
    ff: int = 0                      # dense
    expert: ExpertArgs | None = None
    router: RouterArgs | None = None
    shared: ExpertArgs | None = None


class LayerArgs(base.BaseModelArgs):
    type: str
    mixer: MixerArgs
    mlp: MlpArgs | None = None


class NormArgs(base.BaseModelArgs):
    eps: float


class ModelArgs(base.BaseModelArgs):
    architecture: str = "Taduzen"
    layers: list[LayerArgs]
    vocab: int
    width: int
    logit_scale: float
    norm: NormArgs


class Model(LayerStackModel):
    model_type = "taduzen"

    def __init__(self, args: ModelArgs, weights: dict[str, torch.Tensor], dtype: torch.dtype = torch.bfloat16):
        """weights: the checkpoint's tensors on the device (bf16; tables int32).  dtype: bfloat16, or float32 for 32-bit arithmetic throughout."""
        W = args.width

        def get(name: str, *shape: int) -> torch.Tensor:
            t = weights.get(name)
            if t is None:
                raise ValueError(f"{name} is missing from the checkpoint")
            if tuple(t.shape) != shape:
                raise ValueError(f"{name}: expected {list(shape)}, got {list(t.shape)}")
            return t

        def norm(name: str) -> Norm:
            return Norm(_ffi.PIE_NORM_DYN_TANH, float(get(name + ".alpha").float().item()), pad(get(name, W).float()[None], 1, up8(W))[0], pad(get(name + ".b", W).float()[None], 1, up8(W))[0])

        def pack(w: torch.Tensor) -> torch.Tensor:
            return pack_linear(w, dtype)

        if not args.layers:
            raise ValueError("a model has at least one layer")
        layers = []
        for i, lay in enumerate(args.layers):
            p, m, ff = f"l{i}.", lay.mixer, lay.mlp
            if lay.type != "latent_attention":
                raise ValueError(f"layer {i}: unknown mixer {lay.type!r}")
            H, D, V, R = m.heads, m.dim, m.vdim, m.kv_rank
            q = pad_head_rows(get(p + "mix.q", H * D, W), H, D)
            uk, uv = get(p + "mix.uk", H * D, R), get(p + "mix.uv", H * V, R)
            wo = get(p + "mix.o", W, H * V)
            fields = {
                "pre1": norm(p + "norm1"), "post1": norm(p + "norm1b"), "mixer": _ffi.PIE_MIXER_LATENT,
                "heads": H, "dim": D, "vdim": V, "rank": R, "window": m.mask.size if m.mask is not None else 0, "scale": m.scale, "eps": args.norm.eps,
                "w_in": pack(torch.cat([q, pad(get(p + "mix.dkv", R, W), up8(R), W)])),
                "w_uk": pack(uk.view(H, D, R).transpose(1, 2)),
                "w_uv": pack(uv.view(H, V, R)),
                "w_o": pack(pad_head_columns(wo, H, V)),
                "w_kv": pack(torch.cat([pad_head_rows(uk, H, D), pad_head_rows(uv, H, V)])),
                "c_norm": get(p + "mix.dkv.norm", R).float().contiguous(),
            }
            if ff is not None:
                fields |= {"pre2": norm(p + "norm2"), "post2": norm(p + "norm2b")}
                # (intermediate widths padded to 8 with zero rows and columns: act(0) = 0 for both activations)
                def gated(pfx: str, n: int):
                    n8 = up8(n)
                    return (pack(interleave(pad(get(pfx + "gate", n, W), n8, W), pad(get(pfx + "up", n, W), n8, W))), pack(pad(get(pfx + "down", W, n), W, n8)))

                if ff.kind == "dense":
                    n8 = up8(ff.ff)
                    fields |= {"ff": _ffi.PIE_FF_RELU2, "ff_size": n8, "w_up": pack(pad(get(p + "mlp.up", ff.ff, W), n8, W)),
                               "w_down": pack(pad(get(p + "mlp.down", W, ff.ff), W, n8))}
                elif ff.kind == "moe":
                    E, top = ff.router.experts, ff.router.top
                    experts = [gated(f"{p}mlp.e{e}.", ff.expert.ff) for e in range(E)]
                    fields |= {"ff": _ffi.PIE_FF_TABLE_MOE, "ff_size": up8(ff.expert.ff), "experts": E, "top": top,
                               "table": get(p + "mlp.table", args.vocab, top).to(torch.int32).contiguous(),
                               "w_gate_up": torch.cat([e[0] for e in experts]), "w_expert_down": torch.cat([e[1] for e in experts])}
                    if ff.shared is not None:
                        fields["s_gate_up"], fields["s_down"] = gated(p + "mlp.shared.", ff.shared.ff)
                        fields |= {"shared_size": up8(ff.shared.ff), "shared_gate": pad(get(p + "mlp.shared.sg", 1, W).float(), 1, up8(W))[0]}
                else:
                    raise ValueError(f"layer {i}: unknown feed-forward {ff.kind!r}")
            layers.append(fields)
        super().__init__(args, dtype, W, args.vocab, args.logit_scale, layers, get("embed", args.vocab, W).to(torch.bfloat16).contiguous(),
                         pack(get("head", args.vocab, W)), norm("final.norm"))
