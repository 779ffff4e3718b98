"""Kodupel on the device against the plain oracle (oracle/kodupel_oracle.py), in float32 and bfloat16."""
import json
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import kodupel_util as ku
from oracle import kodupel_oracle as orc

pytestmark = pytest.mark.gpu
TOL = {torch.float32: 3e-5, torch.bfloat16: 0.04}
BOTH = pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["f32", "bf16"])


def build(cfg, w, dtype, pages=64, slots=32):
    """A model whose pages and state slots hold old numbers, as used ones do."""
    from proxy_inference_engine_amd.models.kodupel import Model, ModelArgs
    m = Model(ModelArgs(**cfg), {k: v.cuda() for k, v in w.items()}, dtype=dtype)
    pool = m.enable_paged_kv(num_pages=pages, max_sequences=slots)
    for s in pool.states:
        if s is not None:
            s.fill_(1e6)
    return m


def whole(m, ids):
    c = m.make_cache()
    out = m.step_portions([(ids, c)], [list(range(len(ids)))]).cpu().numpy()
    c[0].page_manager.release()
    return out


def in_portions(m, ids, cuts):
    c, got = m.make_cache(), []
    for lo, hi in zip([0, *cuts], [*cuts, len(ids)]):
        got.append(m.step_portions([(ids[lo:hi], c)], [list(range(hi - lo))]).cpu().numpy())
    c[0].page_manager.release()
    return np.concatenate(got)


@BOTH
@pytest.mark.parametrize("name", ku.CONFIGS)
def test_whole_prompts(name, dtype):
    cfg = ku.CONFIGS[name]
    w = ku.weights(cfg, seed=3, q_gain=1.5)
    m, wn = build(cfg, w, dtype), ku.as_numpy(w)
    for n in (1, 2, 17, 40, 150):
        ids, want = ku.sequence(cfg, wn, n, seed=n)
        assert ku.err(whole(m, ids), want) < TOL[dtype], n


@BOTH
def test_residual_stream_layer_by_layer(dtype):
    cfg = ku.CONFIGS["mixed"]
    w, want = ku.weights(cfg, seed=4), []
    ids, _ = ku.sequence(cfg, ku.as_numpy(w), 90, layers_out=want)
    got = build(cfg, w, dtype).layer_outputs(ids).cpu().numpy()
    for i, r in enumerate(want):
        assert ku.err(got[i], r) < TOL[dtype], i


@BOTH
@pytest.mark.parametrize("dims", [(8, 8), (24, 40), (64, 8), (100, 128), (72, 72), (128, 100), (160, 192), (200, 136), (256, 256), (264, 16), (40, 300)], ids=str)
def test_every_head_width_class(dims, dtype):
    """Prompts, a portion behind them, and decoded tokens; heads too wide for the matrix cores take the vector ALU."""
    cfg = ku.config([(ku.attention(heads=4, kv_heads=2, dim=dims[0], vdim=dims[1]), None)])
    w = ku.weights(cfg, seed=5, q_gain=2.0)
    ids = ku.tokens(cfg, 330)
    want = orc.forward(cfg, ku.as_numpy(w), ids)
    assert ku.err(in_portions(build(cfg, w, dtype), ids, [180, 325, 328, 329]), want) < TOL[dtype]


@pytest.mark.parametrize("heads", [(1, 1), (7, 7), (7, 1), (12, 3), (48, 1), (40, 40), (130, 2)], ids=str)
def test_every_grouping(heads):
    cfg = ku.config([(ku.attention(heads=heads[0], kv_heads=heads[1], dim=24, vdim=16), None)])
    w = ku.weights(cfg, seed=6, q_gain=2.0)
    ids = ku.tokens(cfg, 300)
    want = orc.forward(cfg, ku.as_numpy(w), ids)
    assert ku.err(in_portions(build(cfg, w, torch.bfloat16), ids, [200, 250, 256, 297, 298, 299]), want) < TOL[torch.bfloat16]


@BOTH
@pytest.mark.parametrize("size", [(1, 8, 4), (3, 16, 16), (2, 17, 1), (2, 32, 33), (3, 40, 8), (1, 64, 64), (2, 96, 24), (1, 128, 100), (2, 200, 5), (1, 256, 16)], ids=str)
def test_every_delta_size_class(size, dtype):
    """(heads, dim, rank) in prompts, portions and decoded tokens, with states that forget fast and states that forget little."""
    cfg = ku.config([(ku.delta(heads=size[0], dim=size[1], rank=size[2]), None)], width=72)
    for memory, removal in ((-2.0, 0.0), (-7.0, -3.0), (3.0, 4.0)):
        w = ku.weights(cfg, seed=7, memory=memory, removal=removal)
        m, ids = build(cfg, w, dtype), ku.tokens(cfg, 200)
        want = orc.forward(cfg, ku.as_numpy(w), ids)
        assert ku.err(whole(m, ids), want) < TOL[dtype], memory
        assert ku.err(in_portions(m, ids, [3, 19, 36, 116, 180, 181, 182, 198]), want) < TOL[dtype], memory


@pytest.mark.parametrize("size", [(1, 1, 1), (4, 2, 3)], ids=str)
def test_tiny_delta_heads(size):
    """32-bit only: the direction of so short an output vector is decided by rounding too often in 16."""
    cfg = ku.config([(ku.delta(heads=size[0], dim=size[1], rank=size[2]), None)], width=72)
    w, ids = ku.weights(cfg, seed=7), ku.tokens(cfg, 100)
    want = orc.forward(cfg, ku.as_numpy(w), ids)
    got = in_portions(build(cfg, w, torch.float32), ids, [3, 36, 97, 98])
    d = np.abs(got - want).max(-1)
    assert np.median(d) < 1e-5 and (d > 1e-3).mean() < 0.03


@BOTH
@pytest.mark.parametrize("n", [2, 15, 16, 17, 31, 32, 33, 47, 48, 64, 65, 79, 80, 95, 129])
def test_delta_runs_of_every_length(n, dtype):
    """Runs that end inside, at and just behind a chunk, twice in a row."""
    cfg = ku.config([(ku.delta(heads=2, dim=24, rank=6), None)], width=72)
    w, ids = ku.weights(cfg, seed=8, memory=-4.0, removal=-1.0), ku.tokens(cfg, 2 * n + 1)
    want = orc.forward(cfg, ku.as_numpy(w), ids)
    assert ku.err(in_portions(build(cfg, w, dtype), ids, [n, 2 * n]), want) < TOL[dtype]


@BOTH
def test_a_state_remembers(dtype):
    """One early token decides the output far behind it: decay and removal nearly off, every later key orthogonal to its key.  Losing, clearing or mixing up
    the state at any cut would lose it."""
    D, W, V = 16, 48, 30
    cfg = ku.config([(ku.delta(heads=1, dim=D, rank=4), None)], width=W, vocab=V, scale=1.0)
    w = ku.weights(cfg, seed=9, memory=-14.0, removal=-14.0)
    x = w["embed"].float()
    back = torch.linalg.pinv(x)                               # W x V: rows of the embedding -> unit vectors of the token
    g = torch.Generator().manual_seed(2)
    k, r = torch.zeros(D, W), torch.zeros(D, W)
    k[0] = 3 * back[:, 0]                                     # channel 0: the key of token 0 alone, asked for by every token
    k[1:] = 0.05 * torch.randn(D - 1, V, generator=g) @ back.T
    r[0] = back.sum(1)
    r[1:] = 0.05 * torch.randn(D - 1, V, generator=g) @ back.T
    w["l0.mix.k"], w["l0.mix.r"], w["l0.mix.w2"] = k.to(torch.bfloat16), r.to(torch.bfloat16), torch.zeros_like(w["l0.mix.w2"])
    wn = ku.as_numpy(w)
    m, tol = build(cfg, w, dtype), TOL[dtype] if dtype == torch.float32 else 0.08
    for at in (0, 15, 16, 63, 64):
        ids = np.random.default_rng(at).integers(1, V, 300).astype(np.int32)
        ids[at] = 0
        want = orc.forward(cfg, wn, ids)
        other = ids.copy()
        other[at] = 1
        assert ku.err(orc.forward(cfg, wn, other)[200:], want[200:]) > 0.5      # it is remembered
        assert ku.err(whole(m, ids), want) < tol, at
        assert ku.err(in_portions(m, ids, [40, 42, 130, 145, 146, 290, 291, 292]), want) < tol, at


@BOTH
def test_wider_layers_and_longer_prompts(dtype):
    """Several row and column tiles everywhere, experts with many rows, and one pass of long and short runs together."""
    cfg = ku.config([(ku.attention(heads=8, kv_heads=4, dim=64, vdim=64, dims=32), ku.moe(ff=270, experts=4, top=2)), (ku.delta(heads=5, dim=64, rank=40), None),
                     (ku.attention(kv_from=0, heads=8, kv_heads=4, dim=64, vdim=64, dims=32), ku.moe(ff=72, experts=12, top=5))], width=328, vocab=600)
    w = ku.weights(cfg, seed=17)
    m, wn = build(cfg, w, dtype), ku.as_numpy(w)
    todo = [ku.sequence(cfg, wn, n, seed=n, lead=0.003 if dtype == torch.bfloat16 else 0) for n in (700, 5, 130, 66, 1, 63)]
    caches = [m.make_cache() for _ in todo]
    for cut in (0.6, 1.0):   # the second pass continues every cache
        entries, rows = [], []
        for (t, want), c in zip(todo, caches):
            lo, hi = c[0].offset, max(int(len(t) * cut), 1)
            if hi > lo:
                entries.append((t[lo:hi], c))
                rows.append(want[lo:hi])
        got = m.step_portions(entries, [list(range(len(r))) for r in rows]).cpu().numpy()
        at = 0
        for r in rows:
            assert ku.err(got[at:at + len(r)], r) < TOL[dtype], len(r)
            at += len(r)


@BOTH
def test_prompt_equals_token_by_token(dtype):
    cfg = ku.CONFIGS["mixed"]
    w = ku.weights(cfg, seed=6, q_gain=1.5)
    m = build(cfg, w, dtype)
    ids, want = ku.sequence(cfg, ku.as_numpy(w), 135)
    c = m.make_cache()
    got = []
    for t in ids:
        _, _, logits = m.step(torch.tensor([t], dtype=torch.int32), c)   # captured and replayed from the third step on
        got.append(logits.cpu().numpy().copy())
    assert ku.err(np.stack(got), want) < TOL[dtype]


@BOTH
@pytest.mark.parametrize("cut", [2, 3, 7, 16, 31, 64, 65, 100])
def test_portions(cut, dtype):
    cfg = ku.CONFIGS["mixed"]
    w = ku.weights(cfg, seed=7, q_gain=1.5)
    ids, want = ku.sequence(cfg, ku.as_numpy(w), 203)
    assert ku.err(in_portions(build(cfg, w, dtype), ids, list(range(cut, 203, cut))), want) < TOL[dtype]


@BOTH
def test_mixed_batches_reuse_pages_and_slots(dtype):
    """Unequal requests side by side -- portions, single tokens, requests left out of a step -- in a pool so small that pages and slots come back."""
    cfg = ku.CONFIGS["mixed"]
    w, rng = ku.weights(cfg, seed=8, q_gain=1.5), np.random.default_rng(0)
    m, wn = build(cfg, w, dtype, pages=9, slots=4), ku.as_numpy(w)
    todo = [ku.sequence(cfg, wn, int(n), seed=100 + i) for i, n in enumerate((130, 70, 5, 65, 128, 1, 90, 33, 64, 127))]
    live, nxt, used, slots = {}, 0, set(), set()
    while nxt < len(todo) or live:
        pages = sum(-(-len(todo[i][0]) // 64) for i in live)
        while nxt < len(todo) and len(live) < 4 and pages + -(-len(todo[nxt][0]) // 64) <= 9:
            live[nxt] = [m.make_cache(), 0]
            pages += -(-len(todo[nxt][0]) // 64)
            nxt += 1
        step = [i for i in live if rng.random() < 0.8] or list(live)[:1]
        entries, rows = [], []
        for i in step:
            n = 1 if rng.random() < 0.4 else int(rng.integers(1, 100))
            lo = live[i][1]
            part = todo[i][0][lo:lo + n]
            entries.append((part, live[i][0]))
            rows.append((i, lo, len(part)))
        got = m.step_portions(entries, [list(range(n)) for _, _, n in rows]).cpu().numpy()
        at = 0
        for i, lo, n in rows:
            assert ku.err(got[at:at + n], todo[i][1][lo:lo + n]) < TOL[dtype], (i, lo, n)
            at += n
            live[i][1] = lo + n
            used.update(live[i][0][0].page_manager.pages)
            slots.add(live[i][0][0].page_manager.slot)
            if lo + n == len(todo[i][0]):
                live.pop(i)[0][0].page_manager.release()
    assert m._pool.get_num_free_pages() == 9 and m._pool.num_free_slots() == 4 and len(used) <= 9 and slots <= set(range(4))


@BOTH
def test_far_keys(dtype):
    """One token's key outscores every other for every query and decides the output as long as it is read -- at page and block borders, from the token's
    own position on, in prompts and in decoding, through the layer's own cache and through a layer that shares it."""
    W, V, D = 64, 50, 16
    cfg = ku.config([(ku.attention(heads=2, kv_heads=2, dim=D, vdim=16, dims=4, base=50.0, scaling=None, scale=1.0), None),
                     (ku.attention(heads=2, kv_heads=2, dim=D, vdim=16, dims=4, base=50.0, scaling=None, scale=1.0, kv_from=0), None)], width=W, vocab=V, scale=1.0, eps=1e-6)
    w = ku.weights(cfg, seed=9)
    back = torch.linalg.pinv(w["embed"].float())
    k = torch.zeros(2 * D, W)
    for h in (0, D):
        k[h + 8] = 3 * back[:, 0]                      # dimension 8 (not rotated): token 0 alone; dimension 9: everything else
        k[h + 9] = 3 * back[:, 1:].sum(1)
    w["l0.mix.k"], w["l0.mix.k.b"] = k.to(torch.bfloat16), torch.zeros_like(w["l0.mix.k.b"])
    for p in ("l0.", "l1."):
        q = torch.zeros(2 * D, W)
        w[p + "mix.q"] = q.to(torch.bfloat16)
        b = torch.zeros(2 * D)
        b[8] = b[D + 8] = 1.0
        w[p + "mix.q.b"] = b.to(torch.bfloat16)
        w[p + "mix.q.norm"] = torch.ones(D, dtype=torch.bfloat16)
    w["l0.mix.k.norm"] = torch.ones(D, dtype=torch.bfloat16)
    wn, n = ku.as_numpy(w), 300
    m = build(cfg, w, dtype)
    for at in (0, 1, 31, 32, 63, 64, 127, 128, 191):
        ids = np.random.default_rng(at).integers(1, V, n).astype(np.int32)
        ids[at] = 0
        want = orc.forward(cfg, wn, ids)
        other = ids.copy()
        other[at] = 1
        assert ku.err(orc.forward(cfg, wn, other)[at + 1:], want[at + 1:]) > 0.3    # it decides
        assert ku.err(whole(m, ids), want) < TOL[dtype], at
        cuts = sorted({*range(at - 2, at + 3), 295, 296, 297, 298, 299} & set(range(1, n)))
        assert ku.err(in_portions(m, ids, cuts), want) < TOL[dtype], at


@BOTH
def test_the_sink_counts(dtype):
    """Scores around zero and below: at a sequence's first tokens, and where every score is very negative, the one in the denominator decides how large the
    heads are against each other."""
    cfg = ku.config([(ku.attention(heads=4, kv_heads=4, dim=16, vdim=16, scale=1.0), None)], width=64, eps=1e-6)
    w = ku.weights(cfg, seed=10)
    for h, level in enumerate((-2.0, -0.3, 0.4, 2.5)):    # a head's scores: level times the key's first entry
        w["l0.mix.q"][16 * h:16 * h + 16] = 0
        w["l0.mix.q.b"][16 * h:16 * h + 16] = 0
        w["l0.mix.q.b"][16 * h + 15] = level
        w["l0.mix.k.b"][16 * h + 15] = 4.0
    w["l0.mix.q.norm"][:] = 1.0
    wn, ids = ku.as_numpy(w), ku.tokens(cfg, 200)
    want = orc.forward(cfg, wn, ids)
    real = orc.sink_softmax
    orc.sink_softmax = lambda s, mask: (lambda p: p / p.sum(-1, keepdims=True))(real(s, mask))
    try:
        without = orc.forward(cfg, wn, ids)
    finally:
        orc.sink_softmax = real
    assert min(ku.err(without[i:i + 1], want[i:i + 1]) for i in (0, 1, 5, 199)) > 0.1
    m = build(cfg, w, dtype)
    assert ku.err(whole(m, ids), want) < TOL[dtype] and ku.err(in_portions(m, ids, [1, 2, 3, 100, 198, 199]), want) < TOL[dtype]


@BOTH
def test_long_decoding(dtype):
    cfg = ku.CONFIGS["mixed"]
    w = ku.weights(cfg, seed=10, q_gain=1.5)
    m = build(cfg, w, dtype)
    ids, want = ku.sequence(cfg, ku.as_numpy(w), 500, lead=0.003)
    c = m.make_cache()
    m.step_portions([(ids[:20], c)], [[]])
    got = []
    for t in ids[20:]:
        got.append(m.step_batch(torch.tensor([t]), [c])[2].clone())
    assert ku.err(torch.cat(got).cpu().numpy(), want[20:]) < TOL[dtype]


@pytest.mark.parametrize("experts,top", [(1, 1), (2, 2), (64, 8), (65, 1), (130, 7), (300, 12)])
def test_routers_of_every_size(experts, top):
    """32-bit: the same experts as the oracle's, also where scores lie close together, in few rows and in many."""
    cfg = ku.config([(ku.attention(heads=1, kv_heads=1), ku.moe(ff=8, experts=experts, top=top))], width=72)
    w = ku.weights(cfg, seed=11)
    w["l0.mlp.router"] = (torch.randn(experts, 72, generator=torch.Generator().manual_seed(5)) * 0.03).to(torch.bfloat16)
    wn = ku.as_numpy(w)
    m = build(cfg, w, torch.float32)
    for n in (1, 3, 64, 150):
        ids, want = ku.sequence(cfg, wn, n, seed=n, lead=1e-6)
        assert ku.err(whole(m, ids), want) < TOL[torch.float32], n


def test_smooth_routing_in_16_bits():
    """Scores anywhere between 0 and 1, as a trained router's: every row without a close call takes the oracle's experts with its weights."""
    cfg = ku.config([(ku.attention(heads=1, kv_heads=1), ku.moe(ff=24, experts=40, top=4))], width=72)
    w = ku.weights(cfg, seed=19)
    w["l0.mlp.router"] = (torch.randn(40, 72, generator=torch.Generator().manual_seed(5)) * 0.04).to(torch.bfloat16)
    ids, leads = ku.tokens(cfg, 300), []
    want = orc.forward(cfg, ku.as_numpy(w), ids, leads=leads)
    clear = leads[0] > 0.006
    assert clear.sum() > 150
    m = build(cfg, w, torch.bfloat16)
    for got in (whole(m, ids), in_portions(m, ids, list(range(20, 300, 20)))):
        assert ku.err(got[clear], want[clear]) < TOL[torch.bfloat16]


def test_equal_scores_take_the_first_experts():
    cfg = ku.config([(ku.attention(heads=1, kv_heads=1), ku.moe(ff=8, experts=9, top=3))], width=72)
    w = ku.weights(cfg, seed=12)
    w["l0.mlp.router"][:], w["l0.mlp.correction"][:] = 0, 0.25
    ids = ku.tokens(cfg, 20)
    assert ku.err(whole(build(cfg, w, torch.float32), ids), orc.forward(cfg, ku.as_numpy(w), ids)) < TOL[torch.float32]


def test_logits_do_not_depend_on_the_batch():
    """The same request alone and among 20 others: equal to rounding, far below what bf16 itself costs."""
    cfg = ku.CONFIGS["mixed"]
    w = ku.weights(cfg, seed=11)
    m, wn = build(cfg, w, torch.bfloat16, pages=128), ku.as_numpy(w)
    ids, _ = ku.sequence(cfg, wn, 100)
    alone = whole(m, ids)
    caches = [m.make_cache() for _ in range(21)]
    entries = [(ku.tokens(cfg, 3 + 11 * i, seed=i), caches[i]) for i in range(20)] + [(ids, caches[20])]
    got = m.step_portions(entries, [[] for _ in range(20)] + [list(range(100))]).cpu().numpy()
    assert ku.err(got, alone) < 0.02


def test_graph_replays_equal_launches():
    """A captured step replayed many times, with other work and synchronisation between, against the same step as launches."""
    cfg = ku.CONFIGS["mixed"]
    w = ku.weights(cfg, seed=12)
    m = build(cfg, w, torch.bfloat16)
    prompts = [ku.tokens(cfg, n, seed=n) for n in (30, 64, 7)]
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


def test_replayed_steps_follow_their_slots():
    """Two sequences take turns at the same captured step: pages and slots are read at replay, not at capture."""
    cfg = ku.CONFIGS["mixed"]
    w = ku.weights(cfg, seed=18)
    m, wn = build(cfg, w, torch.float32), ku.as_numpy(w)
    todo = [ku.sequence(cfg, wn, 40, seed=s, lead=0) for s in (1, 2)]
    caches = [m.make_cache() for _ in todo]
    for t in range(40):
        for (ids, want), c in zip(todo, caches):
            got = m.step_batch(torch.tensor([ids[t]]), [c])[2].cpu().numpy()
            assert ku.err(got, want[t:t + 1]) < 1e-4, t


def greedy(cfg, wn, prompt, n):
    ids, out = list(prompt), []
    for _ in range(n):
        out.append(int(orc.forward(cfg, wn, ids)[-1].argmax()))
        ids.append(out[-1])
    return out


@pytest.mark.parametrize("options", [{}, {"prefill_chunk": 16}, {"share_prefix": True}, {"mixed": False}], ids=["default", "chunked", "shared_prefix", "separate"])
def test_greedy_generation_through_the_engines(options, tmp_path):
    from proxy_inference_engine_amd import InferenceEngine
    from proxy_inference_engine_amd.cache import PromptCache
    from proxy_inference_engine_amd.engine import BatchedEngine
    cfg = ku.CONFIGS["mixed"]
    w = ku.weights(cfg, seed=13)
    wn, m = ku.as_numpy(w), build(cfg, w, torch.float32)
    common = list(ku.tokens(cfg, 70, seed=50))
    prompts = [common + list(ku.tokens(cfg, n, seed=60 + n)) for n in (3, 20, 41, 9, 1)]
    want = [greedy(cfg, wn, p, 8) for p in prompts]
    eng = BatchedEngine(m, num_pages=14, max_batch=3, **options)
    assert eng.generate([[int(t) for t in p] for p in prompts], 8) == want
    assert eng.pool.num_free_slots() == 4 and eng.pool.get_num_free_pages() == 14
    if not options:
        one = InferenceEngine(model=m)
        one.prompt_cache = PromptCache(directory=tmp_path)
        for p, expect in zip(prompts, want):   # other continuations of a common prefix: the state cannot go back, each starts over
            one.prepare_engine(p, temp=0)
            assert [t for t, _ in one.generate(np.asarray(p), max_completion_tokens=8)] == expect
        longer = prompts[-1] + want[-1] + [5, 6]   # the conversation goes on: everything computed is kept
        ids = list(one.prompt_cache.computed_ids)
        assert ids == [int(t) for t in longer[:len(ids)]] and one.prompt_cache.cache[0].reusable(len(ids)) == len(ids)
        one.prompt_cache.cache_prompt()
        one.prepare_engine(longer, temp=0)
        expect = greedy(cfg, wn, longer, 4)
        assert [t for t, _ in one.generate(np.asarray(longer), max_completion_tokens=4)] == expect
        two = InferenceEngine(model=m)              # the same from a file
        two.prompt_cache = PromptCache(directory=tmp_path)
        two.prepare_engine(ids, temp=0)
        assert two.prompt_cache.cache and [t for t, _ in two.generate(np.asarray(longer), max_completion_tokens=4)] == expect


def test_sampling_uses_the_engines_samplers(tmp_path):
    from proxy_inference_engine_amd import InferenceEngine
    from proxy_inference_engine_amd.cache import PromptCache
    cfg = ku.CONFIGS["mixed"]
    m = build(cfg, ku.weights(cfg, seed=14), torch.bfloat16)
    eng = InferenceEngine(model=m)
    eng.prompt_cache = PromptCache(directory=tmp_path)
    prompt = ku.tokens(cfg, 12)
    eng.prepare_engine(prompt, temp=0.8, top_p=0.9, repetition_penalty=1.2)
    out = [t for t, _ in eng.generate(prompt, max_completion_tokens=6)]
    assert len(out) == 6 and all(0 <= t < cfg["vocab"] for t in out)


def test_prompts_longer_than_a_pass(monkeypatch):
    from proxy_inference_engine_amd.models import layer_stack
    monkeypatch.setattr(layer_stack, "MAX_ROWS", 50)
    cfg = ku.CONFIGS["mixed"]
    w, ids = ku.weights(cfg, seed=15), ku.tokens(cfg, 170)
    m, want = build(cfg, w, torch.float32), orc.forward(cfg, ku.as_numpy(w), ids)
    a, b = m.make_cache(), m.make_cache()
    got = m.step_portions([(ids, a), (ids[:90], b)], [[0, 49, 50, 169], [89]]).cpu().numpy()
    assert ku.err(got, want[[0, 49, 50, 169, 89]]) < TOL[torch.float32]


def test_bad_calls_are_refused():
    cfg = ku.CONFIGS["mixed"]
    w = ku.weights(cfg)
    m = build(cfg, w, torch.bfloat16, pages=3, slots=2)
    a, b, c = (m.make_cache() for _ in range(3))
    with pytest.raises(RuntimeError, match="exhausted"):
        m.step_portions([(ku.tokens(cfg, 200), a)], [[]])
    assert a[0].offset == 0 and m._pool.get_num_free_pages() == 3 and m._pool.num_free_slots() == 2
    m.step_portions([([1, 2], a), ([3], b)], [[], []])
    with pytest.raises(RuntimeError, match="slots"):
        m.step_portions([([1], c)], [[]])
    with pytest.raises(ValueError):
        m.step_batch(torch.tensor([1, 1]), [a, a])
    from proxy_inference_engine_amd.models.kodupel import Model, ModelArgs
    dev = {k: v.cuda() for k, v in w.items()}
    for change in (lambda d: d["layers"][3]["mixer"].update(kv_from=1), lambda d: d["layers"][3]["mixer"].update(kv_from=2), lambda d: d["layers"][0].update(type="other")):
        bad = json.loads(json.dumps(cfg))
        change(bad)
        with pytest.raises(ValueError):
            Model(ModelArgs(**bad), dev)
    with pytest.raises(ValueError, match="missing"):
        Model(ModelArgs(**cfg), {k: v for k, v in dev.items() if k != "l1.mix.w1"})


def test_sharing_layers_cache_nothing():
    cfg = ku.CONFIGS["mixed"]
    m = build(cfg, ku.weights(cfg), torch.bfloat16)
    assert [n > 0 for n in m.row_elems] == [True, False, True, False, False, False]
    assert [n > 0 for n in m.state_floats] == [False, True, False, False, True, False] and m.state_floats[1] == 3 * 24 * 24


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_runner(tmp_path, dtype):
    """bin/trace_run on a checkpoint written to disk: two requests, portions beside single tokens, pages and slots used again."""
    from safetensors.torch import save_file
    cfg = ku.CONFIGS["mixed"]
    w = ku.weights(cfg, seed=16)
    wn = ku.as_numpy(w)
    save_file(w, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    (a, wa), (b, wb) = ku.sequence(cfg, wn, 80, seed=1), ku.sequence(cfg, wn, 66, seed=2)
    L = lambda x: [int(t) for t in x]  # noqa: E731
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": L(a[:50]), "want": [0, 49]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": L(b[:65]), "want": []}, {"id": "a", "tokens": L(a[50:51]), "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": L(b[65:]), "want": [0]}, {"id": "a", "tokens": L(a[51:]), "want": [28]}], "end": ["a", "b"]}]
    steps += [{"step": 3 + i, "entries": [{"id": f"c{i}", "tokens": L(a[:66]), "want": [65]}], "end": [f"c{i}"]} for i in range(5)]
    r = subprocess.run([sys.executable, str(Path(__file__).resolve().parent.parent / "bin" / "trace_run"), "--model", str(tmp_path), "--dtype", dtype, "--out", str(tmp_path),
                        "--max-tokens", "256"], input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(8)]
    for i, want in enumerate(([wa[0], wa[49]], [wa[50]], [wb[65], wa[79]], *[[wa[65]]] * 5)):
        got = np.fromfile(tmp_path / f"{i}.f32", dtype="<f4").reshape(len(want), -1)
        assert ku.err(got, np.stack(want)) < TOL[getattr(torch, dtype)], i
