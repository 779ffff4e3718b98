"""Taduzen: latent attention without positions under a sliding window, Dynamic Tanh norms in front of and behind every sublayer, and feed-forwards that
are dense (squared relu) or mixtures whose experts a table picks by token id, beside a gated shared expert.

config.json lists the layers one by one ("layers"), each with its own sizes; tensors are named l<i>.* (norm1, norm1b, norm2, norm2b, mix.*, mlp.*),
embed, final.norm, head.  The arithmetic runs in the native layer stack (models/layer_stack.py); this file reads the configuration and packs the weights."""
from __future__ import annotations

import torch

from .. import base
from ... import _ffi
from ..layer_stack import LayerStackModel, pack_linear


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


def _pad_rows(w: torch.Tensor, heads: int, n: int) -> torch.Tensor:
    """[heads * n, K] -> [heads, n rounded up to 8, K], zero rows behind each head."""
    n8 = (n + 7) // 8 * 8
    out = torch.zeros(heads, n8, w.shape[1], dtype=w.dtype, device=w.device)
    out[:, :n] = w.view(heads, n, -1)
    return out


def _interleave(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
    return torch.stack([gate, up], dim=-2).flatten(-3, -2)


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

        def norm(name: str) -> tuple:
            return (float(get(name + ".alpha").float().item()), get(name, W).float().contiguous(), get(name + ".b", W).float().contiguous())

        def pack(w: torch.Tensor) -> torch.Tensor:
            return pack_linear(w, dtype)

        layers = []
        for i, lay in enumerate(args.layers):
            p, m, ff = f"l{i}.", lay.mixer, lay.mlp
            if lay.type != "latent_attention":
                raise ValueError(f"layer {i}: unknown mixer {lay.type!r}")
            H, D, V, R = m.heads, m.dim, m.vdim, m.kv_rank
            q = _pad_rows(get(p + "mix.q", H * D, W), H, D)
            uk, uv = get(p + "mix.uk", H * D, R), get(p + "mix.uv", H * V, R)
            wo = get(p + "mix.o", W, H * V)
            fields = {
                "pre1": norm(p + "norm1"), "post1": norm(p + "norm1b"), "mixer": _ffi.PIE_MIXER_LATENT,
                "heads": H, "dim": D, "vdim": V, "rank": R, "window": m.mask.size if m.mask is not None else 0, "scale": m.scale, "eps": args.norm.eps,
                "w_in": pack(torch.cat([q.flatten(0, 1), get(p + "mix.dkv", R, W)])),
                "w_uk": pack(uk.view(H, D, R).transpose(1, 2)),
                "w_uv": pack(uv.view(H, V, R)),
                "w_o": pack(_pad_rows(wo.T, H, V).flatten(0, 1).T),
                "c_norm": get(p + "mix.dkv.norm", R).float().contiguous(),
            }
            if ff is not None:
                fields |= {"pre2": norm(p + "norm2"), "post2": norm(p + "norm2b")}
                if ff.kind == "dense":
                    fields |= {"ff": _ffi.PIE_FF_RELU2, "ff_size": ff.ff, "w_up": pack(get(p + "mlp.up", ff.ff, W)), "w_down": pack(get(p + "mlp.down", W, ff.ff))}
                elif ff.kind == "moe":
                    F, E, top = ff.expert.ff, ff.router.experts, ff.router.top
                    fields |= {
                        "ff": _ffi.PIE_FF_TABLE_MOE, "ff_size": F, "experts": E, "top": top,
                        "table": get(p + "mlp.table", args.vocab, top).to(torch.int32).contiguous(),
                        "w_gate_up": torch.cat([pack(_interleave(get(f"{p}mlp.e{e}.gate", F, W), get(f"{p}mlp.e{e}.up", F, W))) for e in range(E)]),
                        "w_expert_down": torch.cat([pack(get(f"{p}mlp.e{e}.down", W, F)) for e in range(E)]),
                    }
                    if ff.shared is not None:
                        S = ff.shared.ff
                        fields |= {"shared_size": S, "s_gate_up": pack(_interleave(get(p + "mlp.shared.gate", S, W), get(p + "mlp.shared.up", S, W))),
                                   "s_down": pack(get(p + "mlp.shared.down", W, S)),
                                   "shared_gate": get(p + "mlp.shared.sg", 1, W).float().reshape(-1).contiguous()}
                else:
                    raise ValueError(f"layer {i}: unknown feed-forward {ff.kind!r}")
            layers.append(fields)
        super().__init__(args, dtype, W, args.vocab, args.logit_scale, layers, get("embed", args.vocab, W).to(torch.bfloat16).contiguous(),
                         pack(get("head", args.vocab, W)), norm("final.norm"))
