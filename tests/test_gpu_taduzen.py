"""Taduzen on the device against the plain oracle (oracle/taduzen_oracle.py), in float32 and bfloat16."""
import json
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import taduzen_util as tu
from oracle import taduzen_oracle as orc

pytestmark = pytest.mark.gpu
TOL = {torch.float32: 3e-5, torch.bfloat16: 0.04}
BOTH = pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["f32", "bf16"])


def build(cfg, w, dtype, pages=64):
    from proxy_inference_engine_amd.models.taduzen import Model, ModelArgs
    m = Model(ModelArgs(**cfg), {k: v.cuda() for k, v in w.items()}, dtype=dtype)
    m.enable_paged_kv(num_pages=pages)
    return m


def whole(m, ids):
    c = m.make_cache()
    out = m.step_portions([(ids, c)], [list(range(len(ids)))]).cpu().numpy()
    c[0].page_manager.release()
    return out


MIXED = [(tu.latent(heads=3, dim=20, vdim=12, rank=40, window=33), tu.dense(72)), (tu.latent(heads=5, dim=8, vdim=24, rank=100, window=70), tu.moe()),
         (tu.latent(heads=1, dim=40, vdim=40, rank=72, window=None), None), (tu.latent(window=1), tu.moe(ff=20, experts=3, top=3, shared=None)),
         (tu.latent(heads=2, window=64), tu.moe(ff=36, experts=9, top=1, shared=12))]
CONFIGS = {
    "attention_only": tu.config([(tu.latent(), None)]),
    "dense_only": tu.config([(tu.latent(heads=1, window=1), tu.dense(100))], width=72),
    "experts_only": tu.config([(tu.latent(heads=1, window=1), tu.moe(shared=None))]),
    "experts_shared": tu.config([(tu.latent(heads=1, window=1), tu.moe(ff=30, experts=7, top=3, shared=50))], width=88, vocab=333),
    "mixed": tu.config(MIXED, width=112, vocab=251, logit_scale=0.7),
    "odd_sizes": tu.config([(tu.latent(heads=3, dim=9, vdim=5, rank=7, window=11), tu.moe(ff=3, experts=1, top=1, shared=5)),
                            (tu.latent(heads=2, dim=1, vdim=1, rank=3, window=3), tu.dense(13))], width=21, vocab=53, logit_scale=2.5, eps=1e-3),
    "many_heads": tu.config([(tu.latent(heads=70, dim=8, vdim=8, rank=64, window=50), tu.dense())], width=128),
}


@BOTH
@pytest.mark.parametrize("name", CONFIGS)
def test_whole_prompts(name, dtype):
    cfg = CONFIGS[name]
    w = tu.weights(cfg, seed=3, q_gain=2.0)
    m, wn = build(cfg, w, dtype), tu.as_numpy(w)
    for n in (1, 2, 17, 40, 150):
        ids = tu.tokens(cfg, n, seed=n)
        assert tu.err(whole(m, ids), orc.forward(cfg, wn, ids)) < TOL[dtype], n


@BOTH
def test_residual_stream_layer_by_layer(dtype):
    cfg = CONFIGS["mixed"]
    w, ids, want = tu.weights(cfg, seed=4), tu.tokens(cfg, 90), []
    orc.forward(cfg, tu.as_numpy(w), ids, want)
    got = build(cfg, w, dtype).layer_outputs(ids).cpu().numpy()
    for i, r in enumerate(want):
        assert tu.err(got[i], r) < TOL[dtype], i


@pytest.mark.parametrize("rank", [8, 64, 72, 129, 192, 256, 330, 512, 520, 640, 700, 1024, 1040])
def test_every_latent_width_class(rank):
    cfg = tu.config([(tu.latent(heads=6, dim=24, vdim=16, rank=rank, window=75), None)])
    w, ids = tu.weights(cfg, seed=5, q_gain=3.0), tu.tokens(cfg, 140)
    assert tu.err(whole(build(cfg, w, torch.bfloat16), ids), orc.forward(cfg, tu.as_numpy(w), ids)) < TOL[torch.bfloat16]


@pytest.mark.parametrize("dims", [(24, 40), (64, 8), (100, 128), (128, 100), (200, 136), (256, 256), (264, 16)], ids=str)
def test_every_head_width_class(dims):
    """Prompts (keys and values spelled out, up to 256 per head), a portion behind them, and decoded tokens."""
    cfg = tu.config([(tu.latent(heads=3, dim=dims[0], vdim=dims[1], rank=72, window=100), None)])
    w, ids = tu.weights(cfg, seed=5, q_gain=3.0), tu.tokens(cfg, 330)
    m, want = build(cfg, w, torch.bfloat16), orc.forward(cfg, tu.as_numpy(w), ids)
    c, got = m.make_cache(), []
    for lo, hi in ((0, 180), (180, 325), (325, 328), (328, 329), (329, 330)):
        got.append(m.step_portions([(ids[lo:hi], c)], [list(range(hi - lo))]).cpu().numpy())
    assert tu.err(np.concatenate(got), want) < TOL[torch.bfloat16]


@BOTH
def test_wider_layers_and_longer_prompts(dtype):
    """Several row and column tiles everywhere, experts with many rows, and one pass of long and short runs together."""
    cfg = tu.config([(tu.latent(heads=4, dim=64, vdim=64, rank=128, window=257), tu.dense(700)),
                     (tu.latent(heads=9, dim=40, vdim=56, rank=136, window=None), tu.moe(ff=270, experts=4, top=2, shared=300))], width=328, vocab=600)
    w = tu.weights(cfg, seed=17, q_gain=1.5)
    m, wn = build(cfg, w, dtype), tu.as_numpy(w)
    todo = [tu.tokens(cfg, n, seed=n) for n in (700, 5, 130, 66, 1, 63)]
    want = [orc.forward(cfg, wn, t) for t in todo]
    caches = [m.make_cache() for _ in todo]
    for cut in (0.6, 1.0):   # the second pass continues every cache
        entries, rows = [], []
        for t, c in zip(todo, caches):
            lo, hi = c[0].offset, max(int(len(t) * cut), 1)
            if hi > lo:
                entries.append((t[lo:hi], c))
                rows.append((len(rows), t, lo, hi))
        got = m.step_portions(entries, [list(range(hi - lo)) for _, _, lo, hi in rows]).cpu().numpy()
        at = 0
        for _, t, lo, hi in rows:
            k = next(i for i, x in enumerate(todo) if x is t)
            assert tu.err(got[at:at + hi - lo], want[k][lo:hi]) < TOL[dtype], (len(t), lo)
            at += hi - lo


@BOTH
def test_prompt_equals_token_by_token(dtype):
    cfg = CONFIGS["mixed"]
    w, ids = tu.weights(cfg, seed=6, q_gain=2.0), tu.tokens(cfg, 135)
    m, want = build(cfg, w, dtype), orc.forward(cfg, tu.as_numpy(w), ids)
    c = m.make_cache()
    got = []
    for t in ids:
        _, _, logits = m.step(torch.tensor([t], dtype=torch.int32), c)   # captured and replayed from the third step on
        got.append(logits.cpu().numpy().copy())
    assert tu.err(np.stack(got), want) < TOL[dtype]


@BOTH
@pytest.mark.parametrize("cut", [2, 3, 7, 31, 64, 65, 100])
def test_portions(cut, dtype):
    cfg = CONFIGS["mixed"]
    w, ids = tu.weights(cfg, seed=7, q_gain=2.0), tu.tokens(cfg, 203)
    m, want = build(cfg, w, dtype), orc.forward(cfg, tu.as_numpy(w), ids)
    c, got = m.make_cache(), []
    for lo in range(0, len(ids), cut):
        part = ids[lo:lo + cut]
        got.append(m.step_portions([(part, c)], [list(range(len(part)))]).cpu().numpy())
    assert tu.err(np.concatenate(got), want) < TOL[dtype]


@BOTH
def test_mixed_batches_reuse_pages(dtype):
    """Unequal requests side by side -- portions, single tokens, requests left out of a step -- in a pool so small that freed pages come back."""
    cfg = CONFIGS["mixed"]
    w, wn, rng = tu.weights(cfg, seed=8, q_gain=2.0), None, np.random.default_rng(0)
    m, wn = build(cfg, w, dtype, pages=9), tu.as_numpy(w)
    todo = [tu.tokens(cfg, int(n), seed=100 + i) for i, n in enumerate((130, 70, 5, 65, 128, 1, 90, 33, 64, 127))]
    want = [orc.forward(cfg, wn, t) for t in todo]
    live, nxt, used = {}, 0, set()
    while nxt < len(todo) or live:
        pages = sum(-(-len(todo[i]) // 64) for i in live)
        while nxt < len(todo) and len(live) < 4 and pages + -(-len(todo[nxt]) // 64) <= 9:
            live[nxt] = [m.make_cache(), 0]
            pages += -(-len(todo[nxt]) // 64)
            nxt += 1
        step = [i for i in live if rng.random() < 0.8] or list(live)[:1]
        entries, rows = [], []
        for i in step:
            n = 1 if rng.random() < 0.4 else int(rng.integers(1, 70))
            lo = live[i][1]
            part = todo[i][lo:lo + n]
            entries.append((part, live[i][0]))
            rows.append((i, lo, len(part)))
        got = m.step_portions(entries, [list(range(n)) for _, _, n in rows]).cpu().numpy()
        at = 0
        for i, lo, n in rows:
            assert tu.err(got[at:at + n], want[i][lo:lo + n]) < TOL[dtype], (i, lo, n)
            at += n
            live[i][1] = lo + n
            used.update(live[i][0][0].page_manager.pages)
            if lo + n == len(todo[i]):
                live.pop(i)[0][0].page_manager.release()
    assert m._pool.get_num_free_pages() == 9 and len(used) <= 9


@BOTH
@pytest.mark.parametrize("window", [2, 63, 64, 65, 97, 128, None])
def test_window_edges_and_far_keys(window, dtype):
    """One token's key outscores every other for every query: it decides the output as long as it is visible -- at page borders, up to the last position
    inside the window, not one further -- in prompts and in decoding.  A mistake of one token in the oracle is visible (and only there)."""
    cfg = tu.config([(tu.latent(heads=2, dim=16, vdim=16, rank=32, window=window, scale=1.0), None)], width=64, vocab=50, eps=1e-6)
    w = tu.weights(cfg, seed=9)
    # token 0 alone drives latent direction 0; every query asks for it
    h = torch.tanh(w["l0.norm1.alpha"].float() * w["embed"].float()) * w["l0.norm1"].float() + w["l0.norm1.b"].float()   # [50, 64], full row rank
    back = torch.linalg.pinv(h)
    dkv = 0.3 * torch.randn(32, 64, generator=torch.Generator().manual_seed(1)) / 8
    dkv[0] = 6 * back[:, 0]
    w["l0.mix.dkv"] = dkv.to(torch.bfloat16)
    uk, q = torch.zeros(32, 32), torch.zeros(32, 64)
    uk[0, 0] = uk[16, 0] = 1.0
    q[0] = q[16] = 4 * back.sum(1)
    w["l0.mix.uk"], w["l0.mix.q"] = uk.to(torch.bfloat16), q.to(torch.bfloat16)
    wn, n = tu.as_numpy(w), 300
    m, tol = build(cfg, w, dtype), max(TOL[dtype], 3e-5 if dtype == torch.float32 else 0.12)   # scores of 20: a rounded query moves the weights
    worst_seen = 0.0
    for at in (0, 5, 63, 64, 127, 128):
        ids = np.random.default_rng(at).integers(1, 50, n).astype(np.int32)
        ids[at] = 0
        want = orc.forward(cfg, wn, ids)
        assert tu.err(whole(m, ids), want) < tol, at
        if window is not None:
            edge = at + window            # first position that no longer sees it
            other = json.loads(json.dumps(cfg))
            other["layers"][0]["mixer"]["mask"]["size"] = window + 1
            wrong = orc.forward(other, wn, ids)
            worst_seen = max(worst_seen, tu.err(wrong[edge:edge + 1], want[edge:edge + 1]))
            lo = max(edge - 3, 1)
        else:
            lo = n - 6
        c = m.make_cache()
        m.step_portions([(ids[:lo], c)], [[]])
        for t in range(lo, min(lo + 6, n)):
            got = m.step_portions([(ids[t:t + 1], c)], [[0]]).cpu().numpy()
            assert tu.err(got, want[t:t + 1]) < tol, (at, t)
        c[0].page_manager.release()
    assert window is None or worst_seen > 0.5


@BOTH
def test_long_decoding_past_windows_and_pages(dtype):
    cfg = CONFIGS["mixed"]
    w = tu.weights(cfg, seed=10, q_gain=2.0)
    m, ids = build(cfg, w, dtype), tu.tokens(cfg, 500)
    want = orc.forward(cfg, tu.as_numpy(w), ids)
    c = m.make_cache()
    m.step_portions([(ids[:20], c)], [[]])
    got = []
    for t in ids[20:]:
        got.append(m.step_batch(torch.tensor([t]), [c])[2].clone())
    assert tu.err(torch.cat(got).cpu().numpy(), want[20:]) < TOL[dtype]


def test_logits_do_not_depend_on_the_batch():
    """The same request alone and among 20 others: equal to rounding, far below what bf16 itself costs."""
    cfg = CONFIGS["mixed"]
    w = tu.weights(cfg, seed=11)
    m = build(cfg, w, torch.bfloat16, pages=128)
    ids = tu.tokens(cfg, 100)
    alone = whole(m, ids)
    caches = [m.make_cache() for _ in range(21)]
    entries = [(tu.tokens(cfg, 3 + 11 * i, seed=i), caches[i]) for i in range(20)] + [(ids, caches[20])]
    got = m.step_portions(entries, [[] for _ in range(20)] + [list(range(100))]).cpu().numpy()
    assert tu.err(got, alone) < 0.02


def test_graph_replays_equal_launches():
    """A captured step replayed many times, with other work and synchronisation between, against the same step as launches."""
    cfg = CONFIGS["mixed"]
    w = tu.weights(cfg, seed=12)
    m = build(cfg, w, torch.bfloat16)
    prompts = [tu.tokens(cfg, n, seed=n) for n in (30, 64, 7)]
    runs = []
    for graph in (False, True):
        caches = [m.make_cache() for _ in prompts]
        tok, _, _ = m.prefill_batch([list(p) for p in prompts], caches)
        out = []
        for i in range(12):
            tok, logprobs, logits = m.step_batch(tok, caches, graph=graph)
            if i % 3 == 0:
                torch.zeros(1 << 20, device="cuda").add_(1.0).sum().item()
            out.append((tok.clone(), logits.clone(), logprobs.clone()))
        runs.append(out)
        for c in caches:
            c[0].page_manager.release()
    for (t0, l0, p0), (t1, l1, p1) in zip(*runs):
        assert torch.equal(t0, t1) and torch.equal(l0, l1) and torch.equal(p0, p1)
        assert torch.allclose(p0, torch.log_softmax(l0, -1), atol=1e-5)


def greedy(cfg, wn, prompt, n):
    ids, out = list(prompt), []
    for _ in range(n):
        out.append(int(orc.forward(cfg, wn, ids)[-1].argmax()))
        ids.append(out[-1])
    return out


@pytest.mark.parametrize("options", [{}, {"prefill_chunk": 16}, {"share_prefix": True}, {"mixed": False}], ids=["default", "chunked", "shared_prefix", "separate"])
def test_greedy_generation_through_the_engines(options, tmp_path):
    from proxy_inference_engine_amd import InferenceEngine
    from proxy_inference_engine_amd.engine import BatchedEngine
    cfg = CONFIGS["mixed"]
    w = tu.weights(cfg, seed=13)
    wn, m = tu.as_numpy(w), build(cfg, w, torch.float32)
    common = list(tu.tokens(cfg, 70, seed=50))
    prompts = [common + list(tu.tokens(cfg, n, seed=60 + n)) for n in (3, 20, 41, 9, 1)]
    want = [greedy(cfg, wn, p, 8) for p in prompts]
    eng = BatchedEngine(m, num_pages=14, max_batch=3, **options)
    assert eng.generate([[int(t) for t in p] for p in prompts], 8) == want
    if not options:
        one = InferenceEngine(model=m)
        from proxy_inference_engine_amd.cache import PromptCache
        one.prompt_cache = PromptCache(directory=tmp_path)
        for p, expect in zip(prompts, want):   # each request reuses the common prefix the previous one left in the cache
            one.prepare_engine(p, temp=0)
            got = [t for t, _ in one.generate(np.asarray(p), max_completion_tokens=8)]
            assert got == expect
        one.prompt_cache.cache_prompt()
        ids = list(one.prompt_cache.computed_ids)
        two = InferenceEngine(model=m)
        two.prompt_cache = PromptCache(directory=tmp_path)
        two.prepare_engine(ids, temp=0)
        assert two.prompt_cache.cache and [t for t, _ in two.generate(np.asarray(ids + [1, 2]), max_completion_tokens=4)] == greedy(cfg, wn, ids + [1, 2], 4)


def test_sampling_uses_the_engines_samplers(tmp_path):
    from proxy_inference_engine_amd import InferenceEngine
    from proxy_inference_engine_amd.cache import PromptCache
    cfg = CONFIGS["experts_shared"]
    m = build(cfg, tu.weights(cfg, seed=14), torch.bfloat16)
    eng = InferenceEngine(model=m)
    eng.prompt_cache = PromptCache(directory=tmp_path)
    prompt = tu.tokens(cfg, 12)
    eng.prepare_engine(prompt, temp=0.8, top_p=0.9, repetition_penalty=1.2)
    out = [t for t, _ in eng.generate(prompt, max_completion_tokens=6)]
    assert len(out) == 6 and all(0 <= t < cfg["vocab"] for t in out)


def test_prompts_longer_than_a_pass(monkeypatch):
    from proxy_inference_engine_amd.models import layer_stack
    monkeypatch.setattr(layer_stack, "MAX_ROWS", 50)
    cfg = CONFIGS["mixed"]
    w, ids = tu.weights(cfg, seed=15), tu.tokens(cfg, 170)
    m, want = build(cfg, w, torch.float32), orc.forward(cfg, tu.as_numpy(w), ids)
    a, b = m.make_cache(), m.make_cache()
    got = m.step_portions([(ids, a), (ids[:90], b)], [[0, 49, 50, 169], [89]]).cpu().numpy()
    assert tu.err(got, want[[0, 49, 50, 169, 89]]) < TOL[torch.float32]
    tok, logprobs, logits = m.prefill_batch([list(ids), list(ids[:60])], [m.make_cache(), m.make_cache()])
    assert tu.err(logits.cpu().numpy(), want[[169, 59]]) < TOL[torch.float32] and tok.tolist() == want[[169, 59]].argmax(-1).tolist()


def test_bad_calls_are_refused():
    cfg = CONFIGS["attention_only"]
    m = build(cfg, tu.weights(cfg), torch.bfloat16, pages=2)
    c = m.make_cache()
    with pytest.raises(ValueError):
        m.step_portions([([1, 2], c)], [[2]])
    with pytest.raises(ValueError):
        m.step_portions([([1], c), ([2], c)], [[], []])
    with pytest.raises(RuntimeError, match="exhausted"):
        m.step_portions([(tu.tokens(cfg, 129), c)], [[]])
    assert c[0].offset == 0 and m._pool.get_num_free_pages() == 2


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_runner(tmp_path, dtype):
    """bin/trace_run on a checkpoint written to disk: two requests, portions beside single tokens, pages used again."""
    from safetensors.torch import save_file
    cfg = CONFIGS["mixed"]
    w = tu.weights(cfg, seed=16)
    save_file(w, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    a, b = tu.tokens(cfg, 80, seed=1), tu.tokens(cfg, 66, seed=2)
    L = lambda x: [int(t) for t in x]  # noqa: E731
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": L(a[:50]), "want": [0, 49]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": L(b[:65]), "want": []}, {"id": "a", "tokens": L(a[50:51]), "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": L(b[65:]), "want": [0]}, {"id": "a", "tokens": L(a[51:]), "want": [28]}], "end": ["a", "b"]},
             {"step": 3, "entries": [{"id": "c", "tokens": L(a[:66]), "want": [65]}], "end": ["c"]}]
    r = subprocess.run([sys.executable, str(Path(__file__).resolve().parent.parent / "bin" / "trace_run"), "--model", str(tmp_path), "--dtype", dtype, "--out", str(tmp_path),
                        "--max-tokens", "256"], input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(4)]
    wn = tu.as_numpy(w)
    wa, wb = orc.forward(cfg, wn, a), orc.forward(cfg, wn, b)
    for i, want in enumerate(([wa[0], wa[49]], [wa[50]], [wb[65], wa[79]], [wa[65]])):
        got = np.fromfile(tmp_path / f"{i}.f32", dtype="<f4").reshape(len(want), -1)
        assert tu.err(got, np.stack(want)) < TOL[getattr(torch, dtype)], i
