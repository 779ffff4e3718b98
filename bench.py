#!/usr/bin/env python
"""bench.py -- decode tokens/s of Llama-3-8B int4 g=64, batch 1, on MI355X (BASELINE.json's metric).

    python bench.py [--gpus N] [--steps K] [--warmup W]
    python -m torch.distributed.run --nnodes=1 --nproc-per-node N ... bench.py --gpus N --steps K --warmup W

A "step" = one decode step (one token) through InferenceEngine.generate_step: hipGraph replay of the fused
HIP launch sequence, synthetic random-weight checkpoint (no network), weights and KV cache resident in HBM.
Workload (config.workload): Llama-3-8B-shaped, int4 group 64, bf16 activations, 128-token prompt, greedy.
N > 1: batch-1 decode has no independent units inside one sequence and the 8B model fits one card, so ranks are
independent REPLICAS (one sequence each, no data-path collective): value = sum of tokens over ranks / max time.

Prints ONE JSON line on rank 0 with the driver's contract plus:
  roofline     -- the dominant kernel (gate/up W4S GEMV): algorithmic bytes per launch / mean launch duration,
                  measured here with HIP events on the launch stream, against the 8 TB/s HBM3E peak;
                  `step` = the same fraction for the whole decode step (the north-star figure).
                  `stream_peak` / `frac_of_stream`: the same against a bare streaming read measured in this run (pie_stream_read).
                  `step.floor`: what the launch structure itself costs -- per dependent launch 1.59 us of command-processor time, 0.56 us of
                  workgroup start-up, 0.63 us to publish its output, 1.15 us until the consumer has touched it (the barrier-bit chain of
                  tools/pipeline_probe, profiles/r04_pipeline_probe.txt) -- plus the step's bytes at the stream rate measured in this run;
                  `ms_per_step / floor` says how far the step is from ITS floor, `frac` how far from 8 TB/s.
  tp70b        -- only with --gpus N > 1 on the default workload: after the replicas' timing the same ranks decode ONE Llama-3-70B int4
                  sequence tensor-parallel, once per communicator backend (IPC one-shot, RCCL); `value` stays
                  the replicas figure.
  repetitions  -- 5 repetitions of the K timed steps (the first is `value`): median and min ms per step.
  cpu_baseline -- the CPU oracle (oracle/pie_oracle.c, OpenMP) timed on this box's host cores on a bounded sample, at the GPU run's
                  context (the same 128-token prompt).
  parity       -- the same oracle steps teacher-forced through the HIP model (full 32 layers, V = 128256), outside the timed
                  region: greedy ids where the oracle's top-2 margin exceeds the bound, max / rms logit error in bf16 ulps of
                  the largest logit; the process exits non-zero when it fails.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
import time
from pathlib import Path

ROOT = Path(__file__).resolve().parent
sys.path.insert(0, str(ROOT))

import numpy as np  # noqa: E402
import torch  # noqa: E402

HBM_PEAK_GBPS = 8000.0  # MI355X HBM3E spec (MI355X_MICROARCH.md: 8.0 TB/s spec, ~6.3 TB/s achievable)


def parse():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=128)
    ap.add_argument("--warmup", type=int, default=16)
    ap.add_argument("--prompt", type=int, default=128)
    ap.add_argument("--layers", type=int, default=0, help="debug: override num_hidden_layers (invalidates the metric)")
    ap.add_argument("--no-cpu-baseline", action="store_true")
    ap.add_argument("--cpu-tokens", type=int, default=48)
    ap.add_argument("--kv-splits", type=int, default=0)
    ap.add_argument("--paged", action="store_true", help="KV cache in 64-token pages of one slab (PagedKVCache) instead of contiguous per-layer buffers")
    ap.add_argument("--model", choices=["8b", "70b", "qv", "3b"], default="8b",
                    help="70b: BASELINE.json configs[4]'s model on ONE card (40 GB int4); qv: configs[3]'s Qwen2-VL-7B text tower; 3b: Llama-3.2-3B; not the metric's workload")
    ap.add_argument("--tp", type=int, default=0, help="tensor parallelism over ALL ranks (== --gpus): ONE sequence decoded by the sharded model "
                    "(BASELINE.json configs[4] with --model 70b); strong scaling, value = that sequence's tokens/s")
    ap.add_argument("--tp-backend", choices=["ipc", "rccl"], default="ipc", help="--tp: the communicator behind the fused step's collectives: the one-shot all-reduce over "
                    "IPC-mapped peer memory (default) or RCCL (ncclAllReduce on the launch stream): the comparator for the first run on a real node")
    ap.add_argument("--knob", action="append", default=[], metavar="NAME=VALUE", help="developer: one of the library's test / tuning switches (_ffi.KNOBS) for this run")
    ap.add_argument("--bits", type=int, choices=[2, 4, 6, 8], default=4, help="8 / 6 / 2: MLX int8 / int6 / int2 g=64 weights (W8S / W6S / W2S units; a different workload than the metric's)")
    ap.add_argument("--design", choices=["taduzen", "kodupel", "bezutar", "lagelorn"], help="instead of the metric's workload: prefill and decode throughput of a layer-stack design at sizes that resemble a "
                    "real model's layers, each beside the dense bf16 Llama of equal size (one JSON line; not the BASELINE.json metric)")
    ap.add_argument("--design-only", default="", help="--design: run only the cases whose name contains this (e.g. dense4096/new/decode1)")
    ap.add_argument("--dense", action="store_true", help="BASELINE.json configs[2]: unquantised bf16 weights (a different workload than the metric's)")
    return ap.parse_args()


def _err_eps(got, ref):
    """max |got - ref| and rms(got - ref), in bf16 ulps (2^-8) of the largest / the rms reference logit."""
    eps = 2.0 ** -8
    return (float(np.abs(got - ref).max()) / (eps * float(np.abs(ref).max())),
            float(np.sqrt(np.mean((got - ref) ** 2))) / (eps * float(np.sqrt(np.mean(ref ** 2)))))


def cpu_baseline(cfg, weights_host, n_tokens, model=None, prompt=None, what="Llama-3-8B int4"):
    """Oracle decode tokens/s on the host cores AT THE GPU RUN'S CONTEXT: the benchmark's own prompt (last_only lm_head, untimed), then
    `n_tokens` timed steps, each timed by itself (median and minimum step time reported beside the aggregate).
    With `model` (the HIP model on the same weights) the same steps are then teacher-forced on the GPU and compared:
    the parity gate of the benchmarked configuration itself (full depth, full vocabulary).

    32 layers of random weights amplify every rounding difference (two HIP configurations that differ only in the summation order
    of attention are already 3 ulps apart, scripts/diag_parity_full.py), so the tolerance is not a constant: the same steps also run
    through the oracle in FLOAT32 (same int4 weights, no 16-bit rounding anywhere) and the gate is that the HIP logits are as
    close to that exact-arithmetic result as the bf16 oracle's are (<= 1.5 x its distance, floor 8 ulps), plus identical greedy ids
    wherever the bf16 oracle's top-2 margin exceeds twice its own distance from the float32 result."""
    from oracle import pie_oracle as po

    threads = min(len(os.sched_getaffinity(0)), int(os.environ.get("PIE_CPU_THREADS", "16")))  # the 1-GPU box's CPU share
    po.set_threads(threads)
    orc = po.OracleLlama(cfg, weights_host, "bfloat16")
    cache = [po.OracleKVCache() for _ in orc.layers]
    if prompt is None:
        prompt = np.random.default_rng(1).integers(0, cfg["vocab_size"], 4)
    prompt = np.asarray(prompt, np.int64)
    P = len(prompt)
    t0 = time.perf_counter()
    tok, _ = po.logprobs_argmax(orc.forward(prompt, cache, last_only=True))
    t_prompt = time.perf_counter() - t0
    fed, want, step_s = [], [], []
    for _ in range(n_tokens):
        fed.append(int(tok))
        t0 = time.perf_counter()
        logits = orc.forward(np.array([tok]), cache, last_only=True)
        step_s.append(time.perf_counter() - t0)
        tok, _ = po.logprobs_argmax(logits)
        want.append((np.asarray(logits, np.float32).reshape(-1).copy(), int(tok)))
    dt = float(np.sum(step_s))
    base = {"value": n_tokens / dt, "unit": "tokens/s", "cores": threads, "kind": "port",
            "median_ms_per_step": 1e3 * float(np.median(step_s)), "min_ms_per_step": 1e3 * float(np.min(step_s)),
            "sample": f"oracle/pie_oracle.c (OpenMP, {threads} threads), same synthetic {what} weights, {P}-token prompt ({t_prompt:.1f} s, untimed), "
                      f"then {n_tokens} greedy decode steps at context {P + 1}..{P + n_tokens} ({dt:.1f} s)"}
    if model is None:
        return base, None
    del orc, cache
    w32 = {k: (v if v.dtype == np.uint32 else po.from_bits(v, "bfloat16")) for k, v in weights_host.items()}
    exact = po.OracleLlama(cfg, w32, "float32")
    ecache = [po.OracleKVCache() for _ in exact.layers]
    exact.forward(prompt, ecache, last_only=True)
    gcache = model.make_cache()
    model.step(torch.from_numpy(prompt).to(torch.int32).cuda(), gcache)  # the batched prompt path (MLX's qmm regime from 6 rows, as the oracle's)
    hip_exact = orc_exact = hip_orc = (0.0, 0.0)
    checked = equal = 0
    for t, (ref, otok) in zip(fed, want):
        truth = np.asarray(exact.forward(np.array([t]), ecache, last_only=True), np.float32).reshape(-1)
        gtok, _, glogits = model.step(torch.tensor([t], dtype=torch.int32, device="cuda"), gcache)
        got = glogits.float().cpu().numpy().reshape(-1)
        hip_exact = tuple(max(a, b) for a, b in zip(hip_exact, _err_eps(got, truth)))
        orc_exact = tuple(max(a, b) for a, b in zip(orc_exact, _err_eps(ref, truth)))
        hip_orc = tuple(max(a, b) for a, b in zip(hip_orc, _err_eps(got, ref)))
        top2 = np.sort(ref)[-2:]
        if top2[1] - top2[0] > 2.0 * float(np.abs(ref - truth).max()):  # the bf16 oracle's own choice is not within its rounding noise
            checked += 1
            equal += int(int(gtok.item()) == otok)
    tol = max(1.5 * orc_exact[0], 8.0)
    parity = {"steps": n_tokens, "ids_checked": checked, "ids_equal_where_margin": equal,
              "max_logit_err_eps": hip_orc[0], "max_rms_err_eps": hip_orc[1],
              "vs_float32_oracle": {"hip_max_eps": hip_exact[0], "hip_rms_eps": hip_exact[1], "bf16_oracle_max_eps": orc_exact[0], "bf16_oracle_rms_eps": orc_exact[1]},
              "tolerance_eps": tol, "tolerance_rule": "HIP vs float32 oracle <= max(1.5 x (bf16 oracle vs float32 oracle), 8) ulps of the largest logit",
              "reference": "oracle/pie_oracle.c (parity unpinned: the reference holds no fixture for this path)",
              "min_ids_checked": min(16, n_tokens // 2),
              "ok": bool(equal == checked and checked >= min(16, n_tokens // 2) and hip_exact[0] <= tol)}
    return base, parity


DESIGN_LAYERS = 4
# sizes of real models' layers: 8B-class dense layers, and fine-grained mixtures; `like`: the Llama of equal width, heads and active feed-forward width
DESIGN_SIZES = {
    "taduzen": {
        "dense4096": {"width": 4096, "mixer": {"heads": 32, "dim": 128, "vdim": 128, "kv_rank": 512, "window": 4096}, "mlp": {"ff": 14336},
                      "like": {"hidden_size": 4096, "intermediate_size": 14336, "num_attention_heads": 32, "num_key_value_heads": 8}},
        "moe2048": {"width": 2048, "mixer": {"heads": 16, "dim": 128, "vdim": 128, "kv_rank": 512, "window": 4096},
                    "mlp": {"experts": 64, "top": 6, "ff": 1408, "shared": 2816},
                    "like": {"hidden_size": 2048, "intermediate_size": 11264, "num_attention_heads": 16, "num_key_value_heads": 4}},
    },
    # layers: attention, delta rule, attention on the first layer's keys and values, delta rule
    "kodupel": {
        "wide4096": {"width": 4096, "heads": 32, "kv_heads": 8, "dim": 128, "delta_heads": 32, "rank": 128, "mlp": {"experts": 16, "top": 4, "ff": 3584},
                     "like": {"hidden_size": 4096, "intermediate_size": 14336, "num_attention_heads": 32, "num_key_value_heads": 8}},
        "fine2048": {"width": 2048, "heads": 16, "kv_heads": 4, "dim": 128, "delta_heads": 16, "rank": 64, "mlp": {"experts": 64, "top": 6, "ff": 1408},
                     "like": {"hidden_size": 2048, "intermediate_size": 8448, "num_attention_heads": 16, "num_key_value_heads": 4}},
    },
    # layers: latent attention, minGRU, mLSTM, latent attention on the first layer's latents; `near`: the Taduzen (latent attention without positions, dense squared relu) of equal
    # width, heads, ranks and feed-forward width
    "bezutar": {
        "wide4096": {"width": 4096, "streams": 4, "heads": 32, "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 512, "q_rank": 1536, "mlstm": {"heads": 8, "dim": 256, "vdim": 512},
                     "gru": 4096, "ff": 14336, "near": ("taduzen", {"width": 4096, "mixer": {"heads": 32, "dim": 128, "vdim": 128, "kv_rank": 512, "window": None}, "mlp": {"ff": 14336}}),
                     "like": {"hidden_size": 4096, "intermediate_size": 14336, "num_attention_heads": 32, "num_key_value_heads": 8}},
        "slim2048": {"width": 2048, "streams": 2, "heads": 16, "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 512, "q_rank": 768, "mlstm": {"heads": 8, "dim": 128, "vdim": 256},
                     "gru": 2048, "ff": 8192, "near": ("taduzen", {"width": 2048, "mixer": {"heads": 16, "dim": 128, "vdim": 128, "kv_rank": 512, "window": None}, "mlp": {"ff": 8192}}),
                     "like": {"hidden_size": 2048, "intermediate_size": 8192, "num_attention_heads": 16, "num_key_value_heads": 4}},
    },
    # layers: gated delta rule, attention beside time mixing, twice, each with a feed-forward; `near`: the Kodupel (attention and generalised delta rule, mixtures) of equal width, heads and
    # active feed-forward width
    "lagelorn": {
        "wide4096": {"width": 4096, "heads": 32, "kv_heads": 8, "dim": 128, "chunk": 4096, "delta": {"heads": 32, "kv_heads": 16, "dim": 128, "vdim": 128, "conv": 4}, "time_mix": 32, "rank": 128,
                     "side": 256, "ff": 14336, "near": ("kodupel", "wide4096"),
                     "like": {"hidden_size": 4096, "intermediate_size": 14336, "num_attention_heads": 32, "num_key_value_heads": 8}},
        "slim2048": {"width": 2048, "heads": 16, "kv_heads": 4, "dim": 128, "chunk": 4096, "delta": {"heads": 16, "kv_heads": 16, "dim": 128, "vdim": 256, "conv": 4}, "time_mix": 16, "rank": 64,
                     "side": 128, "ff": 8448, "near": ("kodupel", "fine2048"),
                     "like": {"hidden_size": 2048, "intermediate_size": 8448, "num_attention_heads": 16, "num_key_value_heads": 4}},
    },
}
DESIGN_VOCAB = 32768


def taduzen_checkpoint(size, n_layers, vocab):
    """(config, device weights) of a random Taduzen model of one of its DESIGN_SIZES."""
    W, mx, ff = size["width"], size["mixer"], size["mlp"]
    H, D, V, R = mx["heads"], mx["dim"], mx["vdim"], mx["kv_rank"]
    mixer = {"heads": H, "dim": D, "vdim": V, "kv_rank": R, "scale": D ** -0.5, "mask": mx["window"] and {"size": mx["window"]}}
    mlp = {"kind": "dense", "ff": ff["ff"]} if "experts" not in ff else \
        {"kind": "moe", "expert": {"ff": ff["ff"]}, "router": {"experts": ff["experts"], "top": ff["top"]}, "shared": {"ff": ff["shared"]}}
    cfg = {"architecture": "Taduzen", "vocab": vocab, "width": W, "logit_scale": 1.0, "norm": {"eps": 1e-6},
           "layers": [{"type": "latent_attention", "mixer": mixer, "mlp": mlp}] * n_layers}
    gen = torch.Generator(device="cuda").manual_seed(0)
    w = {}

    def put(name, *shape):
        w[name] = (torch.randn(shape, generator=gen, device="cuda") * shape[-1] ** -0.5).to(torch.bfloat16)

    def norm(name):
        w[name] = torch.ones(W, dtype=torch.bfloat16, device="cuda")
        w[name + ".b"] = torch.zeros(W, dtype=torch.bfloat16, device="cuda")
        w[name + ".alpha"] = torch.tensor(0.5, dtype=torch.bfloat16, device="cuda")
    put("embed", vocab, W)
    for i in range(n_layers):
        p = f"l{i}."
        for n in ("norm1", "norm1b", "norm2", "norm2b"):
            norm(p + n)
        put(p + "mix.q", H * D, W), put(p + "mix.dkv", R, W), put(p + "mix.uk", H * D, R), put(p + "mix.uv", H * V, R), put(p + "mix.o", W, H * V)
        w[p + "mix.dkv.norm"] = torch.ones(R, dtype=torch.bfloat16, device="cuda")
        if "experts" not in ff:
            put(p + "mlp.up", ff["ff"], W), put(p + "mlp.down", W, ff["ff"])
            continue
        for e in [f"e{e}" for e in range(ff["experts"])] + ["shared"]:
            F = ff["shared"] if e == "shared" else ff["ff"]
            put(f"{p}mlp.{e}.gate", F, W), put(f"{p}mlp.{e}.up", F, W), put(f"{p}mlp.{e}.down", W, F)
        put(p + "mlp.shared.sg", 1, W)
        w[p + "mlp.table"] = torch.rand(vocab, ff["experts"], generator=gen, device="cuda").topk(ff["top"], dim=1).indices.to(torch.int32)
    norm("final.norm")
    put("head", vocab, W)
    return cfg, w


def kodupel_checkpoint(size, n_layers, vocab):
    """(config, device weights) of a random Kodupel model of one of its DESIGN_SIZES."""
    W, H, G, D, HD, R, ff = size["width"], size["heads"], size["kv_heads"], size["dim"], size["delta_heads"], size["rank"], size["mlp"]
    mlp = {"kind": "moe", "expert": {"ff": ff["ff"], "limit": 7.0}, "router": {"experts": ff["experts"], "top": ff["top"]}}
    attn = {"heads": H, "kv_heads": G, "dim": D, "vdim": D, "scale": D ** -0.5,
            "rot": {"base": 500000.0, "dims": D // 2, "scaling": {"factor": 4.0, "original": 2048, "fast": 32.0, "slow": 1.0}}}
    layers = [{"type": "general_delta", "mixer": {"heads": HD, "dim": D}, "mlp": mlp} if i % 2 else
              {"type": "attention", "mixer": dict(attn, kv_from=0) if i % 4 else attn, "mlp": mlp} for i in range(n_layers)]
    cfg = {"architecture": "Kodupel", "vocab": vocab, "width": W, "embedding": {"scale": 1.0}, "norm": {"eps": 1e-6}, "layers": layers}
    gen = torch.Generator(device="cuda").manual_seed(0)
    w = {}

    def put(name, *shape, std=None, mean=0.0):
        w[name] = (torch.randn(shape, generator=gen, device="cuda") * (shape[-1] ** -0.5 if std is None else std) + mean).to(torch.bfloat16)
    put("embed", vocab, W, std=1.0)
    for i, lay in enumerate(layers):
        p = f"l{i}."
        put(p + "norm1", W, std=0.02), put(p + "norm2", W, std=0.02)
        if lay["type"] == "attention":
            for n, heads in (("q", H), *((("k", G), ("v", G)) if "kv_from" not in lay["mixer"] else ())):
                put(p + f"mix.{n}", heads * D, W), put(p + f"mix.{n}.b", heads * D, std=0.02)
                if n != "v":
                    put(p + f"mix.{n}.norm", D, std=0.02, mean=1.0)
            put(p + "mix.g", H, W), put(p + "mix.o", W, H * D), put(p + "mix.o.b", W, std=0.02)
        else:
            for n in "rkvga":
                put(p + f"mix.{n}", HD * D, W)
            put(p + "mix.a.b", HD * D, std=1.0), put(p + "mix.w0", HD * D, std=1.0, mean=-3.0), put(p + "mix.w1", R, W), put(p + "mix.w2", HD * D, R)
            put(p + "mix.norm", HD * D, std=0.02, mean=1.0), put(p + "mix.o", W, HD * D)
        for e in range(ff["experts"]):
            put(f"{p}mlp.e{e}.gate", ff["ff"], W), put(f"{p}mlp.e{e}.up", ff["ff"], W), put(f"{p}mlp.e{e}.down", W, ff["ff"])
        put(p + "mlp.router", ff["experts"], W), put(p + "mlp.correction", ff["experts"], std=0.01)
    put("final.norm", W, std=0.02)
    put("head", vocab, W)
    return cfg, w


def bezutar_checkpoint(size, n_layers, vocab):
    """(config, device weights) of a random Bezutar model of one of its DESIGN_SIZES."""
    W, S, H, D, T, U, R, Q, N, F, mem = (size[k] for k in ("width", "streams", "heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank", "gru", "ff", "mlstm"))
    attn = {"heads": H, "dim": D, "rot_dim": T, "vdim": U, "kv_rank": R, "q_rank": Q, "scale": (D + T) ** -0.5,
            "rot": {"base": 500000.0, "dims": T, "scaling": {"factor": 4.0, "original": 2048, "fast": 32.0, "slow": 1.0}}}
    kinds = [("latent_attention", attn), ("mingru", {"width": N}), ("mlstm", dict(mem, gate_cap=15.0)), ("latent_attention", dict(attn, kv_from=0))]
    layers = [{"type": kinds[i % 4][0], "mixer": kinds[i % 4][1], "mlp": {"kind": "dense", "ff": F}} for i in range(n_layers)]
    cfg = {"architecture": "Bezutar", "vocab": vocab, "width": W, "streams": S, "max_positions": 8192, "canon": {"taps": 4}, "norm": {"eps": 1e-6},
           "embedding": {"bigram": {"buckets": 65521, "mul_prev": 31, "mul_cur": 7}}, "layers": layers}
    gen = torch.Generator(device="cuda").manual_seed(0)
    w = {}

    def put(name, *shape, std=None, mean=0.0):
        w[name] = (torch.randn(shape, generator=gen, device="cuda") * (shape[-1] ** -0.5 if std is None else std) + mean).to(torch.bfloat16)
    put("embed", vocab, W, std=1.0), put("bigram", 65522, W, std=0.5), put("pos", 8192, W, std=0.2)
    for i, lay in enumerate(layers):
        p = f"l{i}."
        put(p + "norm1", W, std=0.02), put(p + "norm2", W, std=0.02), put(p + "canon1", W, 4, std=0.2)
        for q in ("hc1.", "hc2."):
            put(p + q + "in", S, std=0.1, mean=1.0 / S), put(p + q + "out", S, std=0.1, mean=1.0), put(p + q + "mix", S, S, std=0.05)
            w[p + q + "mix"] += 0.9 * torch.eye(S, dtype=torch.bfloat16, device="cuda")
        if lay["type"] == "latent_attention":
            put(p + "mix.dq", Q, W), put(p + "mix.dq.norm", Q, std=0.02, mean=1.0), put(p + "mix.uq", H * (D + T), Q), put(p + "mix.uk", H * D, R), put(p + "mix.uv", H * U, R)
            if "kv_from" not in lay["mixer"]:
                put(p + "mix.dkv", R + T, W), put(p + "mix.dkv.norm", R, std=0.02, mean=1.0)
            put(p + "mix.sink", H, std=1.0), put(p + "mix.g", H, W), put(p + "mix.o", W, H * U)
        elif lay["type"] == "mingru":
            put(p + "mix.z", N, W), put(p + "mix.z.b", N, std=1.0, mean=-2.0), put(p + "mix.x", N, W), put(p + "mix.x.b", N, std=0.1), put(p + "mix.g", N, W), put(p + "mix.o", W, N)
        else:
            h, d, v = mem["heads"], mem["dim"], mem["vdim"]
            put(p + "mix.q", h * d, W), put(p + "mix.k", h * d, W), put(p + "mix.v", h * v, W), put(p + "mix.g", h * v, W), put(p + "mix.norm", h * v, std=0.02, mean=1.0)
            put(p + "mix.i", h, W), put(p + "mix.i.b", h, std=0.1), put(p + "mix.f", h, W), put(p + "mix.f.b", h, std=0.1, mean=4.0), put(p + "mix.o", W, h * v)
        put(p + "mlp.up", F, W), put(p + "mlp.down", W, F), put(p + "mlp.act", 2, std=0.1)
    put("final.norm", W, std=0.02)
    put("head", vocab, W)
    return cfg, w


def lagelorn_checkpoint(size, n_layers, vocab):
    """(config, device weights) of a random Lagelorn model of one of its DESIGN_SIZES."""
    W, H, G, D, R, S, F, d, HR = (size[k] for k in ("width", "heads", "kv_heads", "dim", "rank", "side", "ff", "delta", "time_mix"))
    left = {"heads": H, "kv_heads": G, "dim": D, "vdim": D, "scale": D ** -0.5, "bias_max": 128, "mask": {"size": size["chunk"]}}
    kinds = [("delta", d), ("parallel", {"left": left, "right": {"heads": HR, "dim": D}, "left_scale": 0.7, "right_scale": 0.7})]
    layers = [{"type": kinds[i % 2][0], "mixer": kinds[i % 2][1], "mlp": {"kind": "dense", "ff": F}} for i in range(n_layers)]
    cfg = {"architecture": "Lagelorn", "vocab": vocab, "width": W, "max_positions": 8192, "token_side": {"dim": S}, "norm": {"eps": 1e-6}, "postln_alpha": 2.0, "logit_softcap": 30.0, "layers": layers}
    gen = torch.Generator(device="cuda").manual_seed(0)
    w = {}

    def put(name, *shape, std=None, mean=0.0):
        w[name] = (torch.randn(shape, generator=gen, device="cuda") * (shape[-1] ** -0.5 if std is None else std) + mean).to(torch.bfloat16)
    put("embed", vocab, W, std=1.0), put("pos", 8192, W, std=0.2), put("side.embed", vocab, n_layers * S, std=1.0)
    for i, lay in enumerate(layers):
        p = f"l{i}."
        put(p + "norm1", W, std=0.02, mean=1.0), put(p + "norm2", W, std=0.02, mean=1.0), put(p + "side.gate", S, W), put(p + "side.proj", W, S), put(p + "side.norm", W, std=0.02, mean=0.2)
        if lay["type"] == "delta":
            for n, c in (("q", d["kv_heads"] * d["dim"]), ("k", d["kv_heads"] * d["dim"]), ("v", d["heads"] * d["vdim"])):
                put(p + f"mix.{n}", c, W), put(p + f"mix.{n}.conv", c, d["conv"], std=0.5)
            put(p + "mix.g", d["heads"] * d["vdim"], W), put(p + "mix.a", d["heads"], W), put(p + "mix.b", d["heads"], W), put(p + "mix.A_log", d["heads"], std=0.5)
            put(p + "mix.dt_bias", d["heads"], std=1.0, mean=-3.0), put(p + "mix.norm", d["vdim"], std=0.02, mean=1.0), put(p + "mix.o", W, d["heads"] * d["vdim"])
        else:
            q = p + "mix.left."
            put(q + "q", H * D, W), put(q + "q.b", H * D, std=0.02), put(q + "k", G * D, W), put(q + "k.b", G * D, std=0.02), put(q + "q.norm", H * D, std=0.02, mean=1.0)
            put(q + "k.norm", G * D, std=0.02, mean=1.0), put(q + "rel", 32, H, std=0.5), put(q + "sink", H, std=1.0), put(q + "o", W, H * D)
            q = p + "mix.right."
            for n in "rkvgw":
                put(q + "mu." + n, W, std=0.2, mean=0.5)
            for n in "rkvg":
                put(q + n, HR * D, W)
            put(q + "w1", R, W), put(q + "w2", HR * D, R), put(q + "w0", HR * D, std=1.0, mean=-3.0), put(q + "u", HR, D, std=0.3), put(q + "norm", HR * D, std=0.02, mean=1.0), put(q + "o", W, HR * D)
        for n in ("gate", "up"):
            put(p + f"mlp.{n}", F, W), put(p + f"mlp.{n}.b", F, std=0.02)
        put(p + "mlp.down", W, F), put(p + "mlp.down.b", W, std=0.02)
    put("final.norm", W, std=0.02, mean=1.0)
    put("head", vocab, W)
    return cfg, w


def design_bench(args):
    """--design: throughput of a layer-stack design beside the dense bf16 Llama of equal size (and, where one is close, another design), DESIGN_LAYERS layers each."""
    from proxy_inference_engine_amd.models.llama import Model as Llama, ModelArgs as LlamaArgs
    from proxy_inference_engine_amd.models import bezutar, kodupel, lagelorn, taduzen
    from proxy_inference_engine_amd.models.utils import synthetic_checkpoint
    designs = {"taduzen": (taduzen, taduzen_checkpoint), "kodupel": (kodupel, kodupel_checkpoint), "bezutar": (bezutar, bezutar_checkpoint), "lagelorn": (lagelorn, lagelorn_checkpoint)}
    rows = []
    rng = np.random.default_rng(0)

    def timed(fn, n, warm):
        for _ in range(warm):
            fn()
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        for _ in range(n):
            fn()
        torch.cuda.synchronize()
        return 1e3 * (time.perf_counter() - t0) / n

    for name, size in DESIGN_SIZES[args.design].items():
        near = size.get("near")  # another design, and its size (or the name of one)
        for which in ("new", *((near[0],) if near else ()), "llama"):
            if not any(args.design_only in f"{name}/{which}/{c}" for c in ("decode1", "decode8", "decode32", "prefill512", "prefill4096")):
                continue
            if which != "llama":
                design, checkpoint = designs[args.design if which == "new" else which]
                sized = size if which == "new" else DESIGN_SIZES[which][near[1]] if isinstance(near[1], str) else near[1]
                cfg, w = checkpoint(sized, DESIGN_LAYERS, DESIGN_VOCAB)
                model = design.Model(design.ModelArgs(**cfg), w)
            else:
                cfg = dict(size["like"], model_type="llama", num_hidden_layers=DESIGN_LAYERS, vocab_size=DESIGN_VOCAB, rms_norm_eps=1e-6, tie_word_embeddings=False,
                           quantization=None)
                w = synthetic_checkpoint(cfg, dtype=torch.bfloat16)
                model = Llama(LlamaArgs(**cfg), w)
            del w
            torch.cuda.empty_cache()
            model.enable_paged_kv(num_pages=32 * 20, max_blocks=80)
            for L in (512, 4096):
                if args.design_only not in f"{name}/{which}/prefill{L}":
                    continue
                ids = rng.integers(0, DESIGN_VOCAB, L).astype(np.int32)
                dev = torch.from_numpy(ids).cuda()

                def prompt():
                    c = model.make_cache()
                    model.step(dev, c)
                    c[0].page_manager.release()
                ms = timed(prompt, 5, 2)
                rows.append({"size": name, "model": which, "phase": f"prefill {L}", "ms": ms, "tokens_per_s": 1e3 * L / ms})
            for B in (1, 8, 32):
                if args.design_only not in f"{name}/{which}/decode{B}":
                    continue
                ctx = 1024
                caches = [model.make_cache() for _ in range(B)]
                toks = []
                for c in caches:
                    toks.append(model.step(torch.from_numpy(rng.integers(0, DESIGN_VOCAB, ctx).astype(np.int32)).cuda(), c)[0].clone())
                if B == 1:
                    fn = lambda: model.step(None, caches[0])  # noqa: E731
                else:
                    state = [torch.cat(toks)]

                    def fn():
                        state[0] = model.step_batch(state[0], caches)[0]
                ms = timed(fn, args.steps, args.warmup)
                r = {"size": name, "model": which, "phase": f"decode {B} at {ctx}", "ms": ms, "tokens_per_s": 1e3 * B / ms}
                rows.append(r)
                for c in caches:
                    c[0].page_manager.release()
            del model
            torch.cuda.empty_cache()
            print(f"{name} {which} done", file=sys.stderr, flush=True)
    print(json.dumps({"metric": f"{args.design}: prefill and decode throughput, {DESIGN_LAYERS} layers (NOT the BASELINE.json metric)", "dtype": "bf16", "data": "synthetic",
                      "layers": DESIGN_LAYERS, "vocab": DESIGN_VOCAB, "rows": rows}), flush=True)


def tp_shard(full_cfg, tp, rank, dist, backend):
    """This rank's shard of a synthetic tensor-parallel checkpoint, generated directly in the local shapes (the full 70B checkpoint never
    exists anywhere); the replicated tensors (embedding table, norm weights) are rank 0's, broadcast once.  Returns (local config, weights, HipComm)."""
    from proxy_inference_engine_amd.models.utils import synthetic_checkpoint
    from proxy_inference_engine_amd.tp import HipComm, shard_config
    cfg = {k: v for k, v in shard_config(full_cfg, tp).items() if k not in ("tp_world", "tp_vocab_shard")}
    cfg["tie_word_embeddings"] = False
    weights = synthetic_checkpoint(cfg, seed=100 + rank, dtype=torch.bfloat16)
    v_loc = full_cfg["vocab_size"] // tp
    for k in ("weight", "scales", "biases"):
        weights[f"lm_head.{k}"] = weights[f"lm_head.{k}"][:v_loc].contiguous()
    for k, t in weights.items():
        if k.startswith("model.embed_tokens.") or k.endswith("layernorm.weight") or k == "model.norm.weight":
            if dist.get_backend() == "nccl":
                dist.broadcast(t, src=0)
            else:
                h = t.cpu()
                dist.broadcast(h, src=0)
                t.copy_(h)
    return cfg, weights, HipComm(cfg["hidden_size"], backend=backend)


def tp70b_leg(args, rank, world, dist):
    """--gpus N > 1 on the default workload: the first contact with a multi-GPU node should also measure BASELINE.json configs[4] -- ONE
    Llama-3-70B int4 sequence decoded tensor-parallel over all N ranks, once per communicator backend.  Strong scaling: tokens/s of that one
    sequence.  Every failure is recorded, never raised: the replicas line above must survive it."""
    from proxy_inference_engine_amd import InferenceEngine
    from proxy_inference_engine_amd.models.llama import Model, ModelArgs
    from proxy_inference_engine_amd.models.utils import LLAMA3_70B
    out = {"model": "Llama-3-70B-shaped int4 g=64, batch 1", "tp": world, "steps": args.steps, "warmup": args.warmup}
    for backend in ("ipc", "rccl"):
        comm = model = eng = gen = None
        try:
            cfg, weights, comm = tp_shard(dict(LLAMA3_70B), world, rank, dist, backend)
            model = Model(ModelArgs(**cfg), weights, tp=comm)
            del weights
            torch.cuda.empty_cache()
            eng = InferenceEngine(model=model)
            prompt = torch.randint(0, LLAMA3_70B["vocab_size"], (args.prompt,), generator=torch.Generator().manual_seed(1))
            eng.prepare_engine(prompt, temp=0)
            gen = eng.generate_step(prompt)
            for _ in range(1 + args.warmup):
                next(gen)
            torch.cuda.synchronize()
            dist.barrier()
            torch.cuda.synchronize()
            t0 = time.perf_counter()
            for _ in range(args.steps):
                next(gen)
            torch.cuda.synchronize()
            t = torch.tensor([time.perf_counter() - t0], dtype=torch.float64, device="cuda")
            dist.all_reduce(t, op=dist.ReduceOp.MAX)
            dist.barrier()
            elapsed = float(t.item())
            T_mid = args.prompt + 1 + args.warmup + args.steps // 2
            err = comm.status()
            out[backend] = {"tokens_per_s": args.steps / elapsed, "ms_per_step": 1e3 * elapsed / args.steps, "launches_per_step": model.graph_launches(True),
                            "hbm_gbps_per_gpu": model.step_bytes(T_mid, True) * (args.steps / elapsed) / 1e9, "comm_gave_up_at_epoch": err or None}
        except Exception as e:  # noqa: BLE001 -- recorded in the line
            out[backend] = {"error": f"{type(e).__name__}: {e}"[:300]}
        finally:
            del eng, gen, model
            if comm is not None:
                try:
                    comm.close()
                except Exception:  # noqa: BLE001
                    pass
            torch.cuda.empty_cache()
    return out


def main():
    args = parse()
    rank = int(os.environ.get("RANK", "0"))
    local_rank = int(os.environ.get("LOCAL_RANK", "0"))
    world = int(os.environ.get("WORLD_SIZE", "1"))
    if world != args.gpus:
        raise SystemExit(f"--gpus {args.gpus} but WORLD_SIZE={world}: launch with torch.distributed.run --nproc-per-node {args.gpus}")
    n_dev = torch.cuda.device_count()
    if args.design:
        if world > 1:
            raise SystemExit("--design measures one GPU")
        return design_bench(args)
    torch.cuda.set_device(local_rank % max(n_dev, 1))  # one rank per GPU; PIE_BENCH_BACKEND=gloo lets ranks share a card (rehearsal)
    dist = None
    if world > 1:
        import torch.distributed as dist
        os.environ.setdefault("MASTER_ADDR", "127.0.0.1")
        backend = os.environ.get("PIE_BENCH_BACKEND", "nccl")  # "nccl" is RCCL on ROCm
        if backend == "nccl":
            dist.init_process_group("nccl", device_id=torch.device("cuda", local_rank))
        else:
            dist.init_process_group(backend)

    from proxy_inference_engine_amd import InferenceEngine
    from proxy_inference_engine_amd.models.llama import Model, ModelArgs
    from proxy_inference_engine_amd.models.utils import LLAMA3_8B, LLAMA3_70B, LLAMA32_3B, QWEN2VL_7B_TEXT, synthetic_checkpoint

    for kv in args.knob:
        from proxy_inference_engine_amd import _ffi as _knob_ffi
        name, _, value = kv.partition("=")
        _knob_ffi.set_knob(name, int(value))
    cfg = dict({"70b": LLAMA3_70B, "qv": QWEN2VL_7B_TEXT, "3b": LLAMA32_3B}.get(args.model, LLAMA3_8B))
    if args.layers:
        cfg["num_hidden_layers"] = args.layers
    if args.dense:
        cfg["quantization"] = None
    elif args.bits != 4:
        cfg["quantization"] = {"group_size": 64, "bits": args.bits}
    tp = args.tp if args.tp > 1 else 0
    if tp and (tp != world or args.dense or args.bits != 4 or args.paged):
        raise SystemExit("--tp N needs N ranks (--gpus N under torch.distributed.run), int4 weights and contiguous caches")
    comm = None
    if tp:
        full_cfg = cfg
        cfg, weights, comm = tp_shard(full_cfg, tp, rank, dist, args.tp_backend)
    else:
        # heavy-tailed lm_head rows: the parity gate's id comparison needs steps whose greedy token is decided by more than rounding noise
        # (models/utils.py: synthetic_checkpoint); same shapes and bytes, so the timing is that of any Llama-3-8B int4 checkpoint
        weights = synthetic_checkpoint(cfg, seed=0, dtype=torch.bfloat16, lm_head_tail=1.5)
    # the CPU oracle + the teacher-forced parity gate run for every one-card configuration except the 70B model (its oracle step takes 3 s and
    # 120 GB of host memory twice over); dense weights: 8 oracle steps (15 GB per step at 16 bits + 30 GB in float32)
    want_cpu = rank == 0 and world == 1 and not args.no_cpu_baseline and args.model in ("8b", "qv", "3b")
    cpu_tokens = min(args.cpu_tokens, 8) if args.dense else args.cpu_tokens
    weights_host = None
    if want_cpu:  # the oracle reads the same checkpoint, in the reference's on-disk layout, from host memory
        weights_host = {k: (v.cpu().numpy().view(np.uint32) if v.dtype == torch.int32 else v.view(torch.int16).cpu().numpy().view(np.uint16))
                        for k, v in weights.items()}
    model = Model(ModelArgs(**cfg), weights, kv_splits=args.kv_splits, tp=comm)
    del weights
    torch.cuda.empty_cache()

    if args.paged:
        model.enable_paged_kv(num_pages=(args.prompt + args.warmup + args.steps + 2) // 64 + 2)
    eng = InferenceEngine(model=model)
    prompt = torch.randint(0, cfg["vocab_size"], (args.prompt,), generator=torch.Generator().manual_seed(1 if tp else 1 + rank))
    eng.prepare_engine(prompt, temp=0)
    gen = eng.generate_step(prompt)
    next(gen)  # prefill + first token
    for _ in range(args.warmup):
        next(gen)

    def barrier():
        torch.cuda.synchronize()
        if dist is not None:
            dist.barrier()
            torch.cuda.synchronize()

    barrier()
    t0 = time.perf_counter()
    for _ in range(args.steps):
        next(gen)
    torch.cuda.synchronize()
    elapsed = time.perf_counter() - t0
    launches_per_step = model.graph_launches(True)  # kernel nodes of the captured step graph (hipGraphGetNodes), not a formula
    # 5 repetitions, median and min.  `value` stays the driver's contract (the K steps just timed); four more repetitions of
    # the same K steps from the same prompt (the prefix cache makes the re-prefill one token) are reported beside it.
    rep_ms = [1e3 * elapsed / args.steps]
    if world == 1 and not args.layers:
        for _ in range(4):
            gen = eng.generate_step(prompt)
            next(gen)
            for _ in range(args.warmup):
                next(gen)
            torch.cuda.synchronize()
            t1 = time.perf_counter()
            for _ in range(args.steps):
                next(gen)
            torch.cuda.synchronize()
            rep_ms.append(1e3 * (time.perf_counter() - t1) / args.steps)
    if dist is not None:
        t = torch.tensor([elapsed], dtype=torch.float64, device="cuda")
        dist.all_reduce(t, op=dist.ReduceOp.MAX)
        elapsed = float(t.item())
        dist.barrier()
    tokens_per_s = (1 if tp else world) * args.steps / elapsed  # TP: all ranks decode ONE sequence together
    T_mid = args.prompt + 1 + args.warmup + args.steps // 2  # context length in the middle of the timed region
    step_bytes = model.step_bytes(T_mid, True)
    step_gbps = step_bytes * (args.steps / elapsed) / 1e9  # per GPU

    # dominant kernel (gate/up GEMV: 38 % of the step's bytes), timed alone with HIP events on the launch stream,
    # cycling through the layers so every launch streams weights that are not in the 256 MiB Infinity Cache.
    # Events bracket a whole sweep over the layers (back-to-back launches on the launch stream), so the figure is the
    # kernel's steady-state duration -- what rocprofv3 --kernel-trace reports per dispatch -- not launch gaps.
    reps = 8
    n_l = cfg["num_hidden_layers"]
    for li in range(n_l):
        model.launch_kernel("gate_up", li)
    torch.cuda.synchronize()
    ev = [(torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)) for _ in range(reps)]
    for e0, e1 in ev:
        e0.record()
        for li in range(n_l):
            model.launch_kernel("gate_up", li)
        e1.record()
    torch.cuda.synchronize()
    k_ms = float(np.median([a.elapsed_time(b) for a, b in ev])) / n_l
    k_bytes = model.kernel_bytes("gate_up", T_mid)
    k_gbps = k_bytes / (k_ms * 1e-3) / 1e9

    # The measured-stream denominator: a BARE streaming read of 1 GiB shaped like the GEMV's stream (pie_stream_read: one
    # 8-wave workgroup per CU, non-temporal 16-byte loads, nothing computed), timed here with HIP events; best of 5.
    from proxy_inference_engine_amd import _ffi
    sbuf = torch.empty(1 << 30, dtype=torch.uint8, device="cuda")
    sbuf.random_(0, 255)
    lib = _ffi.load()
    _ffi.check(lib.pie_stream_read(sbuf.data_ptr(), sbuf.numel(), _ffi.stream()))
    torch.cuda.synchronize()
    s_ms = []
    for _ in range(5):
        e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        e0.record()
        _ffi.check(lib.pie_stream_read(sbuf.data_ptr(), sbuf.numel(), _ffi.stream()))
        e1.record()
        torch.cuda.synchronize()
        s_ms.append(e0.elapsed_time(e1))
    stream_gbps = sbuf.numel() / (min(s_ms) * 1e-3) / 1e9
    del sbuf

    # HBM bytes per launch of the dominant kernel from the PMC passes over the product step (tools/step_bench under rocprofv3 --pmc,
    # scripts/profile_r03.sh, profiles/README.md).  The file names the library build it was measured on; any other build gets null
    # rather than last round's kernels' traffic.
    traffic = None
    tf = ROOT / "profiles" / "r05_traffic.json"
    if tf.exists() and not args.layers and not args.dense and args.model == "8b" and args.bits == 4:
        rec = json.loads(tf.read_text())
        if rec.get("library") == _ffi.load().pie_version().decode():
            traffic = rec.get("hbm_bytes_per_launch")

    # The floor of the launch structure: a synthetic chain of the step's 161 dependent launches, written as raw AQL packets with
    # the barrier bit and agent fences HIP emits, costs per launch 1.59 us (empty dispatch) + 0.56 (8-wave workgroups, LDS, one barrier) + 0.63
    # (publish the output) + 1.15 (the consumer's first touch of it) = 3.93 us before any weight is streamed, and 1.150 ms with the 8B model's
    # 4.24 GB behind it (tools/pipeline_probe.cpp; profiles/r04_pipeline_probe.txt, "serial: barrier bit, agent fences").  The serial sum below
    # assumes no overlap between those per-launch costs and the stream; the probe's chain overlaps the stream's head with the staging.
    # (The probe chain is the FIVE-launches-per-layer structure, 162 launches.  Since round 5 the 32 / 8 / 128 head geometry runs four per layer -- the
    # attention behind an XCD-local seam of the q|k|v launch -- so `launches` is 130 there and the step may come out below the 162-launch chain.)
    per_launch_us = {"dispatch": 1.59, "workgroup_start": 0.56, "publish": 0.63, "first_touch": 1.15}
    n_launch = launches_per_step if launches_per_step and launches_per_step > 0 else 5 * n_l + 2
    stream_ms = step_bytes / (stream_gbps * 1e9) * 1e3
    launch_ms = n_launch * sum(per_launch_us.values()) * 1e-3
    floor = {"launches": n_launch, "per_launch_us": per_launch_us, "launch_ms": launch_ms, "stream_ms": stream_ms, "serial_sum_ms": launch_ms + stream_ms,
             "probe_chain_ms_8b": 1.150, "probe_chain_launches": 162, "source": "tools/pipeline_probe.cpp, profiles/r04_pipeline_probe.txt (raw-AQL chain of the step's shape); stream term = step bytes / stream_peak of this run",
             "ms_per_step_over_serial_sum": (1e3 * elapsed / args.steps) / (launch_ms + stream_ms)}
    if args.model == "8b" and args.bits == 4 and not args.dense and not args.layers:
        floor["ms_per_step_over_probe_chain"] = (1e3 * elapsed / args.steps) / 1.150

    shape_cfg = full_cfg if tp else cfg
    out = {
        "metric": (f"decode tokens/sec, Llama-3-{args.model.upper()} int4 g=64 batch=1, TP={tp}; achieved HBM GB/s per GPU" if tp else
                   "decode tokens/sec, Llama-3-8B int4 g=64 batch=1; achieved HBM GB/s" if (args.model == "8b" and args.bits == 4 and not args.dense) else
                   f"decode tokens/sec, {'Qwen2-VL-7B text tower' if args.model == 'qv' else 'Llama-3-' + args.model.upper()} "
                   f"{'dense bf16' if args.dense else f'int{args.bits} g=64'} batch=1; achieved HBM GB/s (NOT the BASELINE.json metric's workload)"),
        "value": tokens_per_s, "unit": "tokens/s", "n_gpus": world, "steps": args.steps, "warmup": args.warmup,
        "ms_per_step": 1e3 * elapsed / args.steps, "higher_is_better": True, "scaling": "strong" if tp else "weak", "vs_baseline": None,
        "dtype": "bf16", "dtype_detail": ("bf16 weights" if args.dense else f"uint{args.bits} g=64 weights") + " x bf16 activations, fp32 accumulate (v_dot2c_f32_bf16)", "data": "synthetic",
        "config": {"workload": f"{'Qwen2-VL-7B text tower' if args.model == 'qv' else 'Llama-3-' + args.model.upper()}-shaped (H{shape_cfg['hidden_size']} L{n_l} {shape_cfg['num_attention_heads']}/{shape_cfg['num_key_value_heads']} heads I{shape_cfg['intermediate_size']} V{shape_cfg['vocab_size']}) {'dense bf16' if args.dense else f'int{args.bits} g=64'} greedy decode, batch 1, "
                               f"{args.prompt}-token prompt, context {args.prompt + 1 + args.warmup}..{args.prompt + 1 + args.warmup + args.steps}",
                   "parallelism": f"TP={tp} ({args.tp_backend} collectives)" if tp else ("replicas" if world > 1 else "single GPU"),
                   "launches_per_step": launches_per_step,  # kernel nodes of the captured hipGraph
                   "hipgraph": True, "kv": "paged (64-token pages)" if args.paged else "contiguous"},
        "roofline": {"bound": "hbm", "kernel": "k_w4s_gemv<bf16, rmsnorm, swiglu> (gate/up)", "achieved": k_gbps, "peak": HBM_PEAK_GBPS,
                     "unit": "GB/s", "frac": k_gbps / HBM_PEAK_GBPS, "traffic": traffic, "bytes_per_launch": k_bytes,
                     "ms_per_launch": k_ms,
                     "stream_peak": stream_gbps, "frac_of_stream": k_gbps / stream_gbps,  # measured in this run: pie_stream_read over 1 GiB
                     "step": {"achieved": step_gbps, "frac": step_gbps / HBM_PEAK_GBPS, "frac_of_stream": step_gbps / stream_gbps, "bytes_per_step": step_bytes,
                              "floor": floor}},
        "repetitions": {"ms_per_step": rep_ms, "median_ms_per_step": float(np.median(rep_ms)), "min_ms_per_step": float(np.min(rep_ms))},
    }
    if world > 1 and not tp and args.model == "8b" and args.bits == 4 and not args.dense and not args.layers and not args.paged \
            and os.environ.get("PIE_BENCH_TP70B", "1") != "0":
        del eng, gen, model
        eng = gen = model = None
        torch.cuda.empty_cache()
        out["tp70b"] = tp70b_leg(args, rank, world, dist)
    if rank == 0:
        if want_cpu:
            del eng, gen
            try:
                what = ("Qwen2-VL-7B text tower" if args.model == "qv" else "Llama-3-" + args.model.upper()) + (" dense bf16" if args.dense else f" int{args.bits}")
                out["cpu_baseline"], out["parity"] = cpu_baseline(cfg, weights_host, cpu_tokens, model, prompt=prompt.numpy(), what=what)
            except Exception as e:  # the baseline must never take the GPU number down with it
                out["cpu_baseline"] = {"value": None, "unit": "tokens/s", "cores": 0, "kind": "port", "sample": f"failed: {e}"}
                out["parity"] = {"ok": False, "error": str(e)}
        else:
            out["cpu_baseline"] = {"value": None, "unit": "tokens/s", "cores": 0, "kind": "port",
                                   "sample": "skipped (timed on rank 0 at N=1 only)"}
        print(json.dumps(out), flush=True)
    if comm is not None:
        err = comm.status()
        del eng, gen, model
        comm.close()
        if err:
            raise SystemExit(f"tensor-parallel communicator gave up waiting for a peer (epoch {err})")
    if dist is not None:
        dist.destroy_process_group()
    if rank == 0 and out.get("parity") is not None and not out["parity"].get("ok", False):
        raise SystemExit("parity gate of the benchmarked model FAILED: " + json.dumps(out["parity"]))


if __name__ == "__main__":
    main()
