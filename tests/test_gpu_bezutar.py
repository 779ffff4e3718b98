"""Bezutar on the device against the plain oracle (oracle/bezutar_oracle.py), in float32 and bfloat16."""
import json
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import bezutar_util as bu
from oracle import bezutar_oracle as orc

pytestmark = pytest.mark.gpu
TOL = {torch.float32: 5e-5, torch.bfloat16: 0.04}
BOTH = pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["f32", "bf16"])


def build(cfg, w, dtype, pages=64, slots=32):
    """A model whose pages and state slots hold old numbers, as used ones do."""
    from proxy_inference_engine_amd.models.bezutar import Model, ModelArgs
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
@pytest.mark.parametrize("name", bu.CONFIGS)
def test_whole_prompts(name, dtype):
    cfg = bu.CONFIGS[name]
    w = bu.weights(cfg, seed=4, q_gain=1.5)  # (a seed without outputs that rounding decides)
    m, wn = build(cfg, w, dtype), bu.as_numpy(w)
    for n in (1, 2, 17, 40, 150):
        ids, want = bu.sequence(cfg, wn, n, seed=n)
        assert bu.err(whole(m, ids), want) < TOL[dtype], n


@BOTH
def test_residual_stream_layer_by_layer(dtype):
    cfg = bu.CONFIGS["mixed"]
    w, want = bu.weights(cfg, seed=4), []
    ids = bu.tokens(cfg, 90)
    orc.forward(cfg, bu.as_numpy(w), ids, want)
    m = build(cfg, w, dtype)
    for got in (m.layer_outputs(ids).cpu().numpy(), m.layer_outputs(ids[:30]).cpu().numpy()):
        for i, r in enumerate(want):
            assert bu.err(got[i], r[:got.shape[1]]) < TOL[dtype], i


@BOTH
@pytest.mark.parametrize("sizes", [(8, 2, 8, 8, 8), (24, 8, 40, 56, 33), (64, 64, 64, 100, 72), (128, 64, 128, 136, 96), (72, 24, 200, 64, 16), (128, 16, 64, 250, 40), (200, 56, 136, 330, 24), (20, 10, 20, 448, 64),
                                   (240, 40, 16, 70, 50), (16, 8, 16, 700, 20), (12, 4, 12, 1100, 9)], ids=str)
def test_every_latent_size_class(sizes, dtype):
    """(dim, rot_dim, vdim, kv_rank, q_rank): prompts, portions behind them, decoded tokens; heads too wide to be spelled out, and latents too wide for the matrix cores."""
    D, T, V, R, Q = sizes
    cfg = bu.config([(bu.latent(heads=3, dim=D, rot_dim=T, vdim=V, kv_rank=R, q_rank=Q), None)])
    w = bu.weights(cfg, seed=5, q_gain=2.0)
    ids = bu.tokens(cfg, 330)
    want = orc.forward(cfg, bu.as_numpy(w), ids)
    assert bu.err(in_portions(build(cfg, w, dtype), ids, [180, 325, 328, 329]), want) < TOL[dtype]


@BOTH
def test_rotation_of_a_part(dtype):
    """Fewer rotated numbers than the shared key part has: the others pass unchanged."""
    cfg = bu.config([(bu.latent(rot_dim=16, rot_dims=6), None), (bu.latent(rot_dim=16, rot_dims=6, kv_from=0), None), (bu.latent(rot_dim=8, rot_dims=0), None)])
    w = bu.weights(cfg, seed=6, q_gain=2.0)
    ids = bu.tokens(cfg, 200)
    want = orc.forward(cfg, bu.as_numpy(w), ids)
    assert bu.err(in_portions(build(cfg, w, dtype), ids, [130, 198, 199]), want) < TOL[dtype]


@pytest.mark.parametrize("heads", [1, 2, 31, 33, 48, 130])
def test_every_number_of_heads(heads):
    cfg = bu.config([(bu.latent(heads=heads, dim=8, rot_dim=8, vdim=8), None)])
    w = bu.weights(cfg, seed=6, q_gain=2.0)
    ids = bu.tokens(cfg, 300)
    want = orc.forward(cfg, bu.as_numpy(w), ids)
    assert bu.err(in_portions(build(cfg, w, torch.bfloat16), ids, [200, 250, 256, 297, 298, 299]), want) < TOL[torch.bfloat16]


@BOTH
@pytest.mark.parametrize("size", [(1, 8, 8), (2, 17, 5), (3, 32, 33), (2, 40, 64), (1, 64, 16), (2, 96, 40), (1, 130, 30), (1, 256, 48), (1, 300, 20), (2, 520, 16), (3, 8, 300)], ids=str)
def test_every_mlstm_size_class(size, dtype):
    """(heads, dim, vdim) in prompts, portions and decoded tokens, with states that forget fast and states that forget little, gates around zero and large ones."""
    cfg = bu.config([(bu.mlstm(*size), None)], width=72)
    for memory, entry in ((3.0, 0.0), (9.0, 2.0), (-3.0, -4.0)):
        w = bu.weights(cfg, seed=7, memory=memory, entry=entry)
        m, ids = build(cfg, w, dtype), bu.tokens(cfg, 200)
        want = orc.forward(cfg, bu.as_numpy(w), ids)
        assert bu.err(whole(m, ids), want) < TOL[dtype], memory
        assert bu.err(in_portions(m, ids, [3, 19, 36, 116, 180, 181, 182, 198]), want) < TOL[dtype], memory


@BOTH
def test_mlstm_floor_of_the_denominator(dtype):
    """Weak input gates and a head norm whose epsilon counts: the size of a head's output is what the floor under its denominator makes it."""
    cfg = bu.config([(bu.mlstm(), None), (bu.mlstm(heads=2, dim=40, vdim=16), None)], eps=0.3)
    w = bu.weights(cfg, seed=7, memory=1.0, entry=-2.0)
    ids = bu.tokens(cfg, 200)
    want = orc.forward(cfg, bu.as_numpy(w), ids)
    m = build(cfg, w, dtype)
    assert bu.err(whole(m, ids), want) < TOL[dtype] and bu.err(in_portions(m, ids, [1, 2, 5, 100, 101, 199]), want) < TOL[dtype]


@BOTH
@pytest.mark.parametrize("n", [2, 7, 8, 15, 16, 17, 31, 33, 63, 64, 65, 79, 127, 128, 129])
def test_recurrent_runs_of_every_length(n, dtype):
    """Runs that end inside, at and just behind a chunk, twice in a row."""
    cfg = bu.config([(bu.mlstm(heads=2, dim=24, vdim=40), None), (bu.mingru(40), None)], width=72)
    w, ids = bu.weights(cfg, seed=8, memory=5.0, update=-4.0), bu.tokens(cfg, 2 * n + 1)
    want = orc.forward(cfg, bu.as_numpy(w), ids)
    assert bu.err(in_portions(build(cfg, w, dtype), ids, [n, 2 * n]), want) < TOL[dtype]


@BOTH
@pytest.mark.parametrize("width", [1, 2, 7, 8, 129, 300, 1030])
def test_every_mingru_width(width, dtype):
    cfg = bu.config([(bu.mingru(width), None)], width=72)
    for update in (-5.0, 0.0, 4.0):
        w = bu.weights(cfg, seed=9, update=update)
        m, ids = build(cfg, w, dtype), bu.tokens(cfg, 150)
        want = orc.forward(cfg, bu.as_numpy(w), ids)
        assert bu.err(whole(m, ids), want) < TOL[dtype], update
        assert bu.err(in_portions(m, ids, [2, 9, 73, 74, 148]), want) < TOL[dtype], update


@BOTH
@pytest.mark.parametrize("mixer", ["mlstm", "mingru"])
def test_a_state_remembers(mixer, dtype):
    """One early token decides the output far behind it: nothing is forgotten, and later tokens hardly enter.  Losing, clearing or mixing up the state at any cut would lose it."""
    W, V, N = 48, 30, 16
    cfg = bu.config([(bu.mlstm(heads=1, dim=N, vdim=N, gate_cap=12.0) if mixer == "mlstm" else bu.mingru(N), None)], width=W, vocab=V)
    w = bu.plain(bu.weights(cfg, seed=9), cfg)
    w["l0.norm1"].zero_()
    x = w["embed"].double()
    back = torch.linalg.pinv((x / x.pow(2).mean(-1, keepdim=True).sqrt())).float()   # W x V: rows of the normed embedding -> unit vectors of the token
    first, others = back[:, 0], back[:, 1:].sum(1)
    if mixer == "mlstm":   # the input gate opens for token 0 only, whose value every later query asks for
        w["l0.mix.i"], w["l0.mix.i.b"] = (20.0 * first - 20.0 * others)[None].to(torch.bfloat16), torch.zeros(1, dtype=torch.bfloat16)
        w["l0.mix.f"], w["l0.mix.f.b"] = torch.zeros(1, W, dtype=torch.bfloat16), torch.full((1,), 40.0, dtype=torch.bfloat16)
        w["l0.mix.q"] = ((first + others) * torch.ones(N, 1)).to(torch.bfloat16)
        w["l0.mix.k"] = ((first + others) * (1 + torch.arange(N)[:, None] / N)).to(torch.bfloat16)
    else:
        w["l0.mix.z"], w["l0.mix.z.b"] = ((12.0 * first - 12.0 * others) * torch.ones(N, 1)).to(torch.bfloat16), torch.zeros(N, dtype=torch.bfloat16)
    wn = bu.as_numpy(w)
    m = build(cfg, w, dtype)
    for at in (0, 15, 16, 63, 64):
        ids = np.random.default_rng(at).integers(1, V, 300).astype(np.int32)
        ids[at] = 0
        want = orc.forward(cfg, wn, ids)
        other = ids.copy()
        other[at] = 1
        assert bu.err(orc.forward(cfg, wn, other)[200:], want[200:]) > 0.1      # it is remembered
        assert bu.err(whole(m, ids), want) < TOL[dtype], at
        assert bu.err(in_portions(m, ids, [40, 42, 130, 145, 146, 290, 291, 292]), want) < TOL[dtype], at


@BOTH
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 8, 9, 16])
def test_convolutions_of_every_length(taps, dtype):
    """Taps that outweigh the row itself, in runs shorter and longer than the filter, behind portions of every small size, and decoded."""
    cfg = bu.config([(bu.mingru(24), None), (bu.latent(), dense_or_none(taps))], width=76, taps=taps)
    w = bu.weights(cfg, seed=10)
    for n in ("l0.canon1", "l1.canon1"):
        w[n][:, 0] += 2.0
    ids = bu.tokens(cfg, 140)
    want = orc.forward(cfg, bu.as_numpy(w), ids)
    m = build(cfg, w, dtype)
    assert bu.err(whole(m, ids), want) < TOL[dtype]
    assert bu.err(in_portions(m, ids, [1, 3, 5, 8, 12, 13, 14, 30, 62, 64, 129, 130, 131, 138]), want) < TOL[dtype]
    assert bu.err(in_portions(m, ids, list(range(1, 140))), want) < TOL[dtype]


def dense_or_none(taps):
    return bu.dense(24) if taps % 2 else None


@BOTH
@pytest.mark.parametrize("streams", [1, 2, 3, 4, 5, 9, 16])
def test_every_number_of_streams(streams, dtype):
    cfg = bu.config([(bu.mingru(24), bu.dense(40)), (bu.mlstm(), None), (bu.latent(), bu.dense(24))], width=76, streams=streams)
    w, want = bu.weights(cfg, seed=11), []
    ids = bu.tokens(cfg, 100)
    logits = orc.forward(cfg, bu.as_numpy(w), ids, want)
    m = build(cfg, w, dtype)
    got = m.layer_outputs(ids).cpu().numpy()
    assert all(bu.err(a, b) < TOL[dtype] for a, b in zip(got, want))
    assert bu.err(in_portions(m, ids, [70, 75, 76, 77]), logits) < TOL[dtype]


@BOTH
@pytest.mark.parametrize("width", [5, 20, 50, 260, 300, 1028, 2052, 4100])
def test_every_width(width, dtype):
    cfg = bu.config([(bu.mingru(16), bu.dense(24))], width=width, vocab=40, positions=90)
    w = bu.weights(cfg, seed=12)
    ids = bu.tokens(cfg, 80)
    want = orc.forward(cfg, bu.as_numpy(w), ids)
    m = build(cfg, w, dtype)
    assert bu.err(whole(m, ids), want) < TOL[dtype] and bu.err(in_portions(m, ids, [70, 75, 76]), want) < TOL[dtype]


@pytest.mark.parametrize("bigram", [(1, 3, 5), (7, 1, 0), (509, 1000003, 999983), (1000, 1 << 40, (1 << 41) + 3)], ids=str)
def test_bigrams_cross_every_cut(bigram):
    """The previous token is carried over portions, decoded tokens and other sequences' steps, also where the products leave 32 bits."""
    cfg = bu.config([(bu.mingru(8), None)], width=40, bigram=bigram)
    w = bu.weights(cfg, seed=13)
    w["bigram"] *= 3
    wn = bu.as_numpy(w)
    m = build(cfg, w, torch.float32)
    (a, wa), (b, wb) = bu.sequence(cfg, wn, 60, seed=1), bu.sequence(cfg, wn, 60, seed=2)
    assert bu.err(whole(m, a), wa) < 5e-5 and bu.err(in_portions(m, a, [1, 2, 4, 20, 21, 40]), wa) < 5e-5
    ca, cb, got = m.make_cache(), m.make_cache(), []
    for lo, hi in ((0, 1), (1, 2), (2, 4), (4, 30), (30, 31), (31, 60)):
        got.append(m.step_portions([(a[lo:hi], ca), (b[lo:hi], cb)], [list(range(hi - lo))] * 2).cpu().numpy())
    for part, (lo, hi) in zip(got, ((0, 1), (1, 2), (2, 4), (4, 30), (30, 31), (31, 60))):
        assert bu.err(part[:hi - lo], wa[lo:hi]) < 5e-5 and bu.err(part[hi - lo:], wb[lo:hi]) < 5e-5, lo


@BOTH
def test_wider_layers_and_longer_prompts(dtype):
    """Several row and column tiles everywhere, and one pass of long and short runs together."""
    cfg = bu.config([(bu.latent(heads=8, dim=64, rot_dim=32, vdim=64, kv_rank=192, q_rank=160), bu.dense(700)), (bu.mlstm(heads=5, dim=64, vdim=96), bu.dense(300)), (bu.mingru(700), None),
                     (bu.latent(heads=8, dim=64, rot_dim=32, vdim=64, kv_rank=192, q_rank=160, kv_from=0), bu.dense(72))], width=328, vocab=600, positions=800)
    w = bu.weights(cfg, seed=17)
    m, wn = build(cfg, w, dtype), bu.as_numpy(w)
    todo = [bu.sequence(cfg, wn, n, seed=n) for n in (700, 5, 130, 66, 1, 63)]
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
            assert bu.err(got[at:at + len(r)], r) < TOL[dtype], len(r)
            at += len(r)


@BOTH
def test_prompt_equals_token_by_token(dtype):
    cfg = bu.CONFIGS["mixed"]
    w = bu.weights(cfg, seed=6, q_gain=1.5)
    m = build(cfg, w, dtype)
    ids, want = bu.sequence(cfg, bu.as_numpy(w), 135)
    c = m.make_cache()
    got = []
    for t in ids:
        _, _, logits = m.step(torch.tensor([t], dtype=torch.int32), c)   # captured and replayed from the third step on
        got.append(logits.cpu().numpy().copy())
    assert bu.err(np.stack(got), want) < TOL[dtype]


@BOTH
@pytest.mark.parametrize("cut", [2, 3, 7, 16, 31, 64, 65, 100])
def test_portions(cut, dtype):
    cfg = bu.CONFIGS["mixed"]
    w = bu.weights(cfg, seed=7, q_gain=1.5)
    ids, want = bu.sequence(cfg, bu.as_numpy(w), 203)
    assert bu.err(in_portions(build(cfg, w, dtype), ids, list(range(cut, 203, cut))), want) < TOL[dtype]


@BOTH
def test_mixed_batches_reuse_pages_and_slots(dtype):
    """Unequal requests side by side -- portions, single tokens, requests left out of a step -- in a pool so small that pages and slots come back."""
    cfg = bu.CONFIGS["mixed"]
    w, rng = bu.weights(cfg, seed=8, q_gain=1.5), np.random.default_rng(0)
    m, wn = build(cfg, w, dtype, pages=9, slots=4), bu.as_numpy(w)
    todo = [bu.sequence(cfg, wn, int(n), seed=100 + i) for i, n in enumerate((130, 70, 5, 65, 128, 1, 90, 33, 64, 127))]
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
            assert bu.err(got[at:at + n], todo[i][1][lo:lo + n]) < TOL[dtype], (i, lo, n)
            at += n
            live[i][1] = lo + n
            used.update(live[i][0][0].page_manager.pages)
            slots.add(live[i][0][0].page_manager.slot)
            if lo + n == len(todo[i][0]):
                live.pop(i)[0][0].page_manager.release()
    assert m._pool.get_num_free_pages() == 9 and m._pool.num_free_slots() == 4 and len(used) <= 9 and slots <= set(range(4))


def lone_token_keys(w, p, cfg, heads, mx):
    """Attention weights under which token 0's unrotated key outscores every other for every query, and its value differs from all others'."""
    W, D, T, V, R, Q = cfg["width"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"], mx["q_rank"]
    x = w["embed"].double()
    back = torch.linalg.pinv((x / x.pow(2).mean(-1, keepdim=True).sqrt())).float()
    if mx.get("kv_from") is None:
        dkv = torch.zeros(R + T, W)
        dkv[0], dkv[1] = 3 * back[:, 0], 3 * back[:, 1:].sum(1)
        w[p + "dkv"] = dkv.to(torch.bfloat16)
        w[p + "dkv.norm"] = torch.ones(R, dtype=torch.bfloat16)
    dq = torch.zeros(Q, W)
    dq[0] = back.sum(1)
    w[p + "dq"], w[p + "dq.norm"] = dq.to(torch.bfloat16), torch.ones(Q, dtype=torch.bfloat16)
    uq, uk = torch.zeros(heads, D + T, Q), torch.zeros(heads, D, R)
    uq[:, 2, 0], uk[:, 2, 0] = 1.0, 1.0
    w[p + "uq"], w[p + "uk"] = uq.flatten(0, 1).to(torch.bfloat16), uk.flatten(0, 1).to(torch.bfloat16)


@BOTH
def test_far_keys(dtype):
    """One token's key outscores every other for every query and decides the output as long as it is read -- at page and block borders, from the token's
    own position on, in prompts and in decoding, through the layer's own cache and through a layer that shares it."""
    kw = dict(heads=2, dim=16, rot_dim=4, vdim=16, kv_rank=12, q_rank=8, scale=0.6, scaling=None, base=50.0)
    cfg = bu.config([(bu.latent(**kw), None), (bu.latent(kv_from=0, **kw), None)], width=64, vocab=50, eps=1e-6)
    w = bu.plain(bu.weights(cfg, seed=9), cfg)
    for i in range(2):
        w[f"l{i}.norm1"].zero_()
        lone_token_keys(w, f"l{i}.mix.", cfg, 2, cfg["layers"][i]["mixer"])
        w[f"l{i}.mix.sink"].zero_()
    w["l0.hc1.out"].zero_()     # (the second layer meets the embedding too)
    wb = {k: v.clone() for k, v in w.items()}
    wb["l0.hc1.out"].fill_(1.0), wb["l1.hc1.out"].zero_()
    n = 300
    for w in (w, wb):
        wn, m = bu.as_numpy(w), build(cfg, w, dtype)
        for at in (0, 1, 31, 32, 63, 64, 127, 128, 191):
            ids = np.random.default_rng(at).integers(1, 50, n).astype(np.int32)
            ids[at] = 0
            want = orc.forward(cfg, wn, ids)
            other = ids.copy()
            other[at] = 1
            assert bu.err(orc.forward(cfg, wn, other)[at + 1:], want[at + 1:]) > 0.05    # it decides
            assert bu.err(whole(m, ids), want) < TOL[dtype], at
            cuts = sorted({*range(at - 2, at + 3), 295, 296, 297, 298, 299} & set(range(1, n)))
            assert bu.err(in_portions(m, ids, cuts), want) < TOL[dtype], at


@BOTH
@pytest.mark.parametrize("level", [-30.0, -2.0, 3.0, 60.0])
def test_the_sinks_count(level, dtype):
    """Sinks far below, around and far above the scores: they decide how large the heads are against each other, at a sequence's first tokens, in prompts and in decoding."""
    cfg = bu.config([(bu.latent(heads=4), None)], width=64, eps=1e-6)
    w = bu.weights(cfg, seed=10)
    w["l0.mix.sink"] = torch.tensor([level, 0.0, -1.0, 2.0], dtype=torch.bfloat16)
    wn, ids = bu.as_numpy(w), bu.tokens(cfg, 200)
    want = orc.forward(cfg, wn, ids)
    without = orc.forward(cfg, wn | {"l0.mix.sink": np.full(4, -1e30)}, ids)
    assert min(bu.err(without[i:i + 1], want[i:i + 1]) for i in (0, 1, 5)) > 0.02
    m = build(cfg, w, dtype)
    assert bu.err(whole(m, ids), want) < TOL[dtype] and bu.err(in_portions(m, ids, [1, 2, 3, 100, 198, 199]), want) < TOL[dtype]


@BOTH
def test_long_decoding(dtype):
    cfg = bu.CONFIGS["mixed"]
    w = bu.weights(cfg, seed=10, q_gain=1.5)
    m = build(cfg, w, dtype)
    ids, want = bu.sequence(cfg, bu.as_numpy(w), 500)
    c = m.make_cache()
    m.step_portions([(ids[:20], c)], [[]])
    got = []
    for t in ids[20:]:
        got.append(m.step_batch(torch.tensor([t]), [c])[2].clone())
    assert bu.err(torch.cat(got).cpu().numpy(), want[20:]) < TOL[dtype]


def test_logits_do_not_depend_on_the_batch():
    """The same request alone and among 20 others: equal to rounding, far below what bf16 itself costs."""
    cfg = bu.CONFIGS["mixed"]
    w = bu.weights(cfg, seed=11)
    m, wn = build(cfg, w, torch.bfloat16, pages=128), bu.as_numpy(w)
    ids, _ = bu.sequence(cfg, wn, 100)
    alone = whole(m, ids)
    caches = [m.make_cache() for _ in range(21)]
    entries = [(bu.tokens(cfg, 3 + 11 * i, seed=i), caches[i]) for i in range(20)] + [(ids, caches[20])]
    got = m.step_portions(entries, [[] for _ in range(20)] + [list(range(100))]).cpu().numpy()
    assert bu.err(got, alone) < 0.02


def test_graph_replays_equal_launches():
    """A captured step replayed many times, with other work and synchronisation between, against the same step as launches."""
    cfg = bu.CONFIGS["mixed"]
    w = bu.weights(cfg, seed=12)
    m = build(cfg, w, torch.bfloat16)
    prompts = [bu.tokens(cfg, n, seed=n) for n in (30, 64, 7)]
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
    cfg = bu.CONFIGS["mixed"]
    w = bu.weights(cfg, seed=18)
    m, wn = build(cfg, w, torch.float32), bu.as_numpy(w)
    todo = [bu.sequence(cfg, wn, 40, seed=s) for s in (1, 2)]
    caches = [m.make_cache() for _ in todo]
    for t in range(40):
        for (ids, want), c in zip(todo, caches):
            got = m.step_batch(torch.tensor([ids[t]]), [c])[2].cpu().numpy()
            assert bu.err(got, want[t:t + 1]) < 1e-4, t


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
    cfg = bu.CONFIGS["mixed"]
    w = bu.weights(cfg, seed=13)
    wn, m = bu.as_numpy(w), build(cfg, w, torch.float32)
    common = list(bu.tokens(cfg, 70, seed=50))
    prompts = [common + list(bu.tokens(cfg, n, seed=60 + n)) for n in (3, 20, 41, 9, 1)]
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
    cfg = bu.CONFIGS["mixed"]
    m = build(cfg, bu.weights(cfg, seed=14), torch.bfloat16)
    eng = InferenceEngine(model=m)
    eng.prompt_cache = PromptCache(directory=tmp_path)
    prompt = bu.tokens(cfg, 12)
    eng.prepare_engine(prompt, temp=0.8, top_p=0.9, repetition_penalty=1.2)
    out = [t for t, _ in eng.generate(prompt, max_completion_tokens=6)]
    assert len(out) == 6 and all(0 <= t < cfg["vocab"] for t in out)


def test_positions_end(tmp_path):
    """A sequence cannot grow beyond the position vectors: passes are refused, the engines stop."""
    from proxy_inference_engine_amd import InferenceEngine
    from proxy_inference_engine_amd.cache import PromptCache
    from proxy_inference_engine_amd.engine import BatchedEngine
    cfg = bu.config([(bu.mingru(16), None)], width=40, positions=20)
    w = bu.weights(cfg, seed=15)
    wn, m = bu.as_numpy(w), build(cfg, w, torch.float32)
    ids, want = bu.sequence(cfg, wn, 20)
    c = m.make_cache()
    with pytest.raises(ValueError, match="20 positions"):
        m.step_portions([(list(ids) + [1], c)], [[]])
    got = m.step_portions([(ids, c)], [list(range(20))]).cpu().numpy()
    assert bu.err(got, want) < 5e-5
    with pytest.raises(ValueError, match="20 positions"):
        m.step_batch(torch.tensor([1]), [c])
    with pytest.raises(ValueError, match="20 positions"):
        BatchedEngine(m, num_pages=4, max_batch=2).generate([list(range(21))], 2)
    prompts = [[int(t) for t in ids[:17]], [int(t) for t in ids], [3]]
    expect = [greedy(cfg, wn, p, n) for p, n in zip(prompts, (4, 1, 8))]
    assert BatchedEngine(m, num_pages=4, max_batch=2).generate(prompts, 8) == expect
    one = InferenceEngine(model=m)
    one.prompt_cache = PromptCache(directory=tmp_path)
    one.prepare_engine(prompts[0], temp=0)
    assert [t for t, _ in one.generate(np.asarray(prompts[0]), max_completion_tokens=8)] == expect[0]


def test_prompts_longer_than_a_pass(monkeypatch):
    from proxy_inference_engine_amd.models import layer_stack
    monkeypatch.setattr(layer_stack, "MAX_ROWS", 50)
    cfg = bu.CONFIGS["mixed"]
    w, ids = bu.weights(cfg, seed=15), bu.tokens(cfg, 170)
    m, want = build(cfg, w, torch.float32), orc.forward(cfg, bu.as_numpy(w), ids)
    a, b = m.make_cache(), m.make_cache()
    got = m.step_portions([(ids, a), (ids[:90], b)], [[0, 49, 50, 169], [89]]).cpu().numpy()
    assert bu.err(got, want[[0, 49, 50, 169, 89]]) < TOL[torch.float32]


def test_bad_models_and_calls_are_refused():
    cfg = bu.CONFIGS["mixed"]
    w = bu.weights(cfg)
    m = build(cfg, w, torch.bfloat16, pages=3, slots=2)
    a, b, c = (m.make_cache() for _ in range(3))
    with pytest.raises(RuntimeError, match="exhausted"):
        m.step_portions([(bu.tokens(cfg, 200), a)], [[]])
    assert a[0].offset == 0 and m._pool.get_num_free_pages() == 3 and m._pool.num_free_slots() == 2
    m.step_portions([([1, 2], a), ([3], b)], [[], []])
    with pytest.raises(RuntimeError, match="slots"):
        m.step_portions([([1], c)], [[]])
    from proxy_inference_engine_amd.models.bezutar import Model, ModelArgs
    dev = {k: v.cuda() for k, v in w.items()}
    for change in (lambda d: d["layers"][3]["mixer"].update(kv_from=1), lambda d: d["layers"][7]["mixer"].update(kv_from=3), lambda d: d["layers"][0].update(type="other"),
                   lambda d: d["layers"][0]["mlp"].update(kind="other"), lambda d: d["layers"][3]["mixer"].update(kv_from=5)):
        bad = json.loads(json.dumps(cfg))
        change(bad)
        with pytest.raises(ValueError):
            Model(ModelArgs(**bad), dev)
    with pytest.raises(ValueError, match="missing"):
        Model(ModelArgs(**cfg), {k: v for k, v in dev.items() if k != "l1.mix.z"})


def test_what_layers_cache():
    cfg = bu.CONFIGS["mixed"]
    m = build(cfg, bu.weights(cfg), torch.bfloat16)
    assert m.row_elems == [48, 0, 0, 0, 0, 40, 0, 0]
    conv = 4 * 112
    assert m.state_floats == [conv + 4, 72 + conv, 3 * (24 * 20 + 24 + 3) + 3 + conv, conv, 2 * (9 * 8 + 12 + 2) + conv, conv, 52 + conv, conv]


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_runner(tmp_path, dtype):
    """bin/trace_run on a checkpoint written to disk: two requests, portions beside single tokens, pages and slots used again."""
    from safetensors.torch import save_file
    cfg = bu.CONFIGS["mixed"]
    w = bu.weights(cfg, seed=16)
    wn = bu.as_numpy(w)
    save_file(w, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    (a, wa), (b, wb) = bu.sequence(cfg, wn, 80, seed=1), bu.sequence(cfg, wn, 66, seed=2)
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
        assert bu.err(got, np.stack(want)) < TOL[getattr(torch, dtype)], i
