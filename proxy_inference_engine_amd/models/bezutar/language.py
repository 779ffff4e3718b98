"""Bezutar: several residual streams (hyper-connections) over mLSTM, minGRU and latent attention layers in any order, each behind a short causal convolution, with
dense xIELU feed-forwards; the embedding is a sum of token, bigram and position vectors.  Latent attention: queries out of a latent of their own, a rotated key part that
all heads share (YaRN scaling), a learned sink and an output gate per head, latents shared between layers.

config.json lists the layers one by one ("layers"), each with its own sizes; tensors are named l<i>.* (norm1, norm2, canon1, hc1.*, hc2.*, mix.*, mlp.*), embed, bigram,
pos, final.norm, head.  The arithmetic runs in the native layer stack (models/layer_stack.py); this file reads the configuration and packs the weights."""
from __future__ import annotations

import math

import torch

from .. import base
from ... import _ffi
from ..layer_stack import Embedding, LayerStackModel, Norm, pack_linear, pad, pad_head_columns, pad_head_rows, up8, yarn_frequencies

DENOMINATOR_EPS = 1e-6   # of an mLSTM head's output
NEGATIVE_SLOPE = 0.5     # what xIELU's second factor has besides its softplus


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
    width: int = 0             # minGRU
    heads: int = 0             # the others
    dim: int = 0
    vdim: int = 0
    gate_cap: float = 0.0      # mLSTM
    q_rank: int = 0            # latent attention, from here on
    kv_rank: int = 0
    rot_dim: int = 0
    scale: float = 0.0
    rot: RotArgs | None = None
    kv_from: int | None = None


class MlpArgs(base.BaseModelArgs):
    kind: str
    ff: int


class LayerArgs(base.BaseModelArgs):
    type: str
    mixer: MixerArgs
    mlp: MlpArgs | None = None


class NormArgs(base.BaseModelArgs):
    eps: float


class CanonArgs(base.BaseModelArgs):
    taps: int


class BigramArgs(base.BaseModelArgs):
    buckets: int
    mul_prev: int
    mul_cur: int


class EmbeddingArgs(base.BaseModelArgs):
    bigram: BigramArgs


class ModelArgs(base.BaseModelArgs):
    architecture: str = "Bezutar"
    layers: list[LayerArgs]
    vocab: int
    width: int
    streams: int
    max_positions: int
    embedding: EmbeddingArgs
    canon: CanonArgs
    norm: NormArgs


class Model(LayerStackModel):
    model_type = "bezutar"

    def __init__(self, args: ModelArgs, weights: dict[str, torch.Tensor], dtype: torch.dtype = torch.bfloat16):
        """weights: the checkpoint's tensors on the device (bf16).  dtype: bfloat16, or float32 for 32-bit arithmetic throughout."""
        W, eps, S, taps = args.width, args.norm.eps, args.streams, args.canon.taps

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

        def table(name: str, rows: int) -> torch.Tensor:
            return get(name, rows, W).to(torch.bfloat16).contiguous()

        def hyper(p: str) -> torch.Tensor:
            return torch.cat([flat(p + "in", S), flat(p + "out", S), flat(p + "mix", S, S).flatten()])

        def latent(p: str, m: MixerArgs) -> dict:
            H, D, V, Q, R, T = m.heads, m.dim, m.vdim, m.q_rank, m.kv_rank, m.rot_dim
            own = m.kv_from is None
            rows = [pad(get(p + "dq", Q, W), up8(Q), W)]
            if own:
                down = get(p + "dkv", R + T, W)
                rows += [pad(down[:R], up8(R), W), pad(down[R:], up8(T), W)]
            rows.append(pad(get(p + "g", H, W), up8(H), W))
            q_norm, up = flat(p + "dq.norm", Q), get(p + "uq", H * (D + T), Q)
            if dtype == torch.bfloat16:  # the norm's weight goes into the matrix behind it: few rows are normed on their way into that product
                q_norm, up = None, (up.float() * q_norm).to(torch.bfloat16)
            up = up.view(H, D + T, Q)
            uk, uv = get(p + "uk", H * D, R), get(p + "uv", H * V, R)
            out = {"mixer": _ffi.PIE_MIXER_LATENT, "heads": H, "dim": D, "vdim": V, "rank": R, "q_rank": Q, "rot_dim": T, "kv_from": -1 if own else m.kv_from, "scale": m.scale,
                   "out_gate": 1, "head_sink": flat(p + "sink", H), "w_in": pack(torch.cat(rows)), "q_norm": q_norm,
                   "w_uq": pack(torch.cat([pad_head_rows(up[:, :D].flatten(0, 1), H, D), pad_head_rows(up[:, D:].flatten(0, 1), H, T)])),
                   "w_uk": pack(uk.view(H, D, R).transpose(1, 2)), "w_uv": pack(uv.view(H, V, R)), "w_kv": pack(torch.cat([pad_head_rows(uk, H, D), pad_head_rows(uv, H, V)])),
                   "w_o": pack(pad_head_columns(get(p + "o", W, H * V), H, V))}
            if own:
                out["c_norm"] = flat(p + "dkv.norm", R)
            if m.rot is not None and m.rot.dims > 0:
                s = m.rot.scaling
                freq, gain = yarn_frequencies(m.rot.dims, m.rot.base, None if s is None else (s.factor, s.original, s.fast, s.slow))
                out |= {"rot_dims": m.rot.dims, "rot_gain": gain, "rot_freq": freq.to(uk.device)}
            return out

        def mlstm(p: str, m: MixerArgs) -> dict:
            H, D, V = m.heads, m.dim, m.vdim
            rows = [pad_head_rows(get(p + "q", H * D, W), H, D), pad_head_rows(get(p + "k", H * D, W), H, D), pad_head_rows(get(p + "v", H * V, W), H, V),
                    pad_head_rows(get(p + "g", H * V, W), H, V), pad(get(p + "i", H, W), up8(H), W), pad(get(p + "f", H, W), up8(H), W)]
            return {"mixer": _ffi.PIE_MIXER_MLSTM, "heads": H, "dim": D, "vdim": V, "kv_from": -1, "scale": D ** -0.5, "gate_cap": m.gate_cap, "unit_eps": DENOMINATOR_EPS,
                    "w_in": pack(torch.cat(rows)), "gate_bias": torch.cat([flat(p + "i.b", H), flat(p + "f.b", H)]), "o_norm": flat(p + "norm", H * V),
                    "w_o": pack(pad_head_columns(get(p + "o", W, H * V), H, V))}

        def mingru(p: str, m: MixerArgs) -> dict:
            N, N8 = m.width, up8(m.width)
            bias = torch.zeros(3, N8, dtype=torch.bfloat16, device=get(p + "z.b", N).device)
            bias[0, :N], bias[1, :N] = get(p + "z.b", N), get(p + "x.b", N)
            return {"mixer": _ffi.PIE_MIXER_MINGRU, "heads": 1, "dim": N, "kv_from": -1, "w_in": pack(torch.cat([pad(get(p + n, N, W), N8, W) for n in "zxg"])),
                    "in_bias": bias, "w_o": pack(get(p + "o", W, N))}

        def dense(p: str, ff: MlpArgs) -> dict:
            F, F8 = ff.ff, up8(ff.ff)  # (padded with zero rows and columns: the activation of zero is zero)
            softplus = lambda z: math.log1p(math.exp(-abs(z))) + max(z, 0.0)  # noqa: E731
            up, down = (softplus(float(z)) for z in get(p + "act", 2).float())
            return {"ff": _ffi.PIE_FF_XIELU, "ff_size": F8, "act_alpha": up, "act_beta": NEGATIVE_SLOPE + down, "w_up": pack(pad(get(p + "up", F, W), F8, W)),
                    "w_down": pack(pad(get(p + "down", W, F), W, F8))}

        if not args.layers:
            raise ValueError("a model has at least one layer")
        mixers = {"mlstm": mlstm, "mingru": mingru, "latent_attention": latent}
        layers = []
        for i, lay in enumerate(args.layers):
            p = f"l{i}."
            if lay.type not in mixers:
                raise ValueError(f"layer {i}: unknown mixer {lay.type!r}")
            conv = torch.zeros(taps, (W + 63) // 64 * 64, dtype=torch.float32, device=get("embed", args.vocab, W).device)
            conv[:, :W] = get(p + "canon1", W, taps).float().T
            fields = {"pre1": norm(p + "norm1"), "eps": eps, "hyper1": hyper(p + "hc1."), "conv": conv, "conv_taps": taps} | mixers[lay.type](p + "mix.", lay.mixer)
            if lay.mlp is not None:
                if lay.mlp.kind != "dense":
                    raise ValueError(f"layer {i}: unknown feed-forward {lay.mlp.kind!r}")
                fields |= {"pre2": norm(p + "norm2"), "hyper2": hyper(p + "hc2.")} | dense(p + "mlp.", lay.mlp)
            layers.append(fields)
        b = args.embedding.bigram
        embedding = Embedding(streams=S, positions=table("pos", args.max_positions), bigram=table("bigram", b.buckets + 1), mul_prev=b.mul_prev, mul_cur=b.mul_cur)
        super().__init__(args, dtype, W, args.vocab, 1.0, layers, table("embed", args.vocab), pack(get("head", args.vocab, W)), norm("final.norm"), embedding=embedding)
