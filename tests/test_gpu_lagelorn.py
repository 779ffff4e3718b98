"""Lagelorn on the device against the plain oracle (oracle/lagelorn_oracle.py), in float32 and bfloat16."""
import json
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import lagelorn_util as lu
from oracle import lagelorn_oracle as orc

pytestmark = pytest.mark.gpu
TOL = {torch.float32: 5e-5, torch.bfloat16: 0.04}
BOTH = pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["f32", "bf16"])


def build(cfg, w, dtype, pages=64, slots=32):
    """A model whose pages and state slots hold old numbers, as used ones do (a page's padding stays zero, so pages are used by a sequence first)."""
    from proxy_inference_engine_amd.models.lagelorn import Model, ModelArgs
    m = Model(ModelArgs(**cfg), {k: v.cuda() for k, v in w.items()}, dtype=dtype)
    pool = m.enable_paged_kv(num_pages=pages, max_sequences=slots)
    c = m.make_cache()
    m.step_portions([(lu.tokens(cfg, min(cfg["max_positions"], 64 * min(pages, 4)), seed=99), c)], [[]])
    c[0].page_manager.release()
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


def both_ways(cfg, w, dtype, n, cuts, seed=1):
    """A whole prompt, and the same in portions and decoded tokens, against the oracle."""
    ids = lu.tokens(cfg, n, seed)
    want = orc.forward(cfg, lu.as_numpy(w), ids)
    m = build(cfg, w, dtype)
    assert lu.err(whole(m, ids), want) < TOL[dtype]
    assert lu.err(in_portions(m, ids, cuts), want) < TOL[dtype]


@BOTH
@pytest.mark.parametrize("name", lu.CONFIGS)
def test_whole_prompts(name, dtype):
    cfg = lu.CONFIGS[name]
    w = lu.weights(cfg, seed=4, q_gain=1.5)
    m, wn = build(cfg, w, dtype), lu.as_numpy(w)
    for n in (1, 2, 17, 40, 150):
        ids, want = lu.sequence(cfg, wn, n, seed=n)
        assert lu.err(whole(m, ids), want) < TOL[dtype], n


@BOTH
def test_residual_stream_layer_by_layer(dtype):
    cfg = lu.CONFIGS["mixed"]
    w, want = lu.weights(cfg, seed=4), []
    ids = lu.tokens(cfg, 90)
    orc.forward(cfg, lu.as_numpy(w), ids, want)
    m = build(cfg, w, dtype)
    for got in (m.layer_outputs(ids).cpu().numpy(), m.layer_outputs(ids[:30]).cpu().numpy()):
        for i, r in enumerate(want):
            assert lu.err(got[i], r[:got.shape[1]]) < TOL[dtype], i


# ------------------------------------------------------------------ gated delta rule
@BOTH
@pytest.mark.parametrize("size", [(1, 1, 8, 8), (2, 1, 17, 5), (3, 3, 32, 33), (4, 2, 64, 64), (2, 2, 40, 130), (1, 1, 130, 30), (2, 1, 100, 256), (1, 1, 200, 72), (1, 1, 256, 16), (2, 2, 24, 300)], ids=str)
def test_every_delta_size_class(size, dtype):
    """(heads, kv_heads, dim, vdim) in prompts, portions and decoded tokens, with states that forget little, some and nearly everything at once."""
    cfg = lu.config([(lu.delta(*size), None)], width=72)
    for decay, spread in ((-6.0, 0.5), (-2.0, 2.0), (6.0, 6.0)):
        w = lu.weights(cfg, seed=7, decay=decay, spread=spread)
        both_ways(cfg, w, dtype, 150, [3, 19, 36, 116, 132, 133, 134])


@BOTH
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 8, 9, 16])
def test_convolutions_of_every_length(taps, dtype):
    """The oldest tap outweighs the others: runs shorter and longer than the filter, behind portions of every small size, and decoded."""
    cfg = lu.config([(lu.delta(heads=4, kv_heads=2, conv=taps), None)], width=76)
    w = lu.weights(cfg, seed=10)
    for n in "qkv":
        w[f"l0.mix.{n}.conv"][:, 0] += 1.0
    ids = lu.tokens(cfg, 140)
    want = orc.forward(cfg, lu.as_numpy(w), ids)
    m = build(cfg, w, dtype)
    assert lu.err(whole(m, ids), want) < TOL[dtype]
    assert lu.err(in_portions(m, ids, [1, 3, 5, 8, 12, 13, 14, 30, 62, 64, 129, 130, 131, 138]), want) < TOL[dtype]
    assert lu.err(in_portions(m, ids, list(range(1, 140))), want) < TOL[dtype]


# ------------------------------------------------------------------ time mixing
@BOTH
@pytest.mark.parametrize("size", [(1, 8, 3), (2, 17, 16), (3, 48, 10), (2, 64, 40), (1, 100, 64), (2, 128, 130), (1, 150, 8), (1, 200, 20), (1, 256, 200)], ids=str)
def test_every_time_mixing_size_class(size, dtype):
    """(heads, dim, rank): decays near one, and decays so small that their quotients leave fp32's range."""
    cfg = lu.config([(lu.parallel(lu.left(heads=2, kv_heads=1, dim=8), lu.right(*size[:2])), None)], width=72)
    for decay, spread in ((-5.0, 0.5), (-1.0, 2.0), (3.0, 3.0)):
        w = lu.weights(cfg, seed=8, decay=decay, spread=spread, rank=size[2])
        both_ways(cfg, lu.only(w, ["right"]), dtype, 150, [3, 19, 36, 116, 132, 133, 134])


@BOTH
def test_time_mixing_alone(dtype, monkeypatch):
    """The stack's mixer without an attention beside it: a layer whose description has the one half only."""
    from proxy_inference_engine_amd import _ffi
    from proxy_inference_engine_amd.models.layer_stack import LayerStackModel, pack_linear, pad_head_columns
    cfg = lu.config([(lu.parallel(lu.left(2, 1, 8), lu.right(3, 20)), lu.dense()), (lu.parallel(lu.left(2, 1, 8), lu.right(3, 20)), None)], width=76)
    w = lu.weights(cfg, seed=8)
    for i in range(2):
        w[f"l{i}.mix.left.o"].zero_()
    real = LayerStackModel.__init__
    keep = ("post1", "post2", "eps", "norm_after", "residual_scale", "w_side_gate", "w_side_proj", "side_norm", "time_mix", "ff", "ff_size", "w_up", "up_bias", "w_down", "down_bias")

    def half(self, args, dtype, width, vocab, scale, layers, *rest, **kw):
        alone = [{k: v for k, v in lay.items() if k in keep} | {"mixer": _ffi.PIE_MIXER_TIME_MIX, "kv_from": -1, "w_o": pack_linear(pad_head_columns(w[f"l{i}.mix.right.o"].cuda(), 3, 20), dtype)}
                 for i, lay in enumerate(layers)]
        real(self, args, dtype, width, vocab, scale, alone, *rest, **kw)
    monkeypatch.setattr(LayerStackModel, "__init__", half)
    both_ways(cfg, w, dtype, 150, [3, 19, 36, 116, 132, 133, 134])


@BOTH
@pytest.mark.parametrize("n", [2, 3, 7, 8, 15, 16, 17, 31, 33, 63, 64, 65, 79])
def test_recurrent_runs_of_every_length(n, dtype):
    """Runs that end inside, at and just behind a chunk, twice in a row; the row in front of a portion is the last one of the portion before."""
    cfg = lu.config([(lu.delta(heads=2, dim=24, vdim=40, conv=4), None), (lu.parallel(lu.left(dim=8), lu.right(2, 40)), None)], width=72)
    w, ids = lu.weights(cfg, seed=8), lu.tokens(cfg, 2 * n + 1)
    want = orc.forward(cfg, lu.as_numpy(w), ids)
    assert lu.err(in_portions(build(cfg, w, dtype), ids, [n, 2 * n]), want) < TOL[dtype]


def token_projection(w, W):
    """[W, vocab]: rows of the embedding -> unit vectors of the token."""
    return torch.linalg.pinv(w["embed"].double()).float()


@BOTH
@pytest.mark.parametrize("mixer", ["delta", "time_mix"])
def test_a_state_remembers(mixer, dtype):
    """One early token decides the output far behind it: nothing is forgotten, and later tokens hardly enter.  Losing, clearing or mixing up the state at any cut would lose it."""
    W, V, N = 48, 30, 16
    cfg = lu.config([(lu.delta(heads=1, dim=N, vdim=N, conv=1) if mixer == "delta" else lu.parallel(lu.left(), lu.right(1, N)), None)], width=W, vocab=V)
    w = lu.only(lu.weights(cfg, seed=9), ["right"])
    back = token_projection(w, W)
    first, others = back[:, 0], back[:, 1:].sum(1)
    q = "l0.mix." if mixer == "delta" else "l0.mix.right."
    ramp = 1 + torch.arange(N)[:, None] / N
    every = ((first + others) * ramp).to(torch.bfloat16)   # the same key and query for every token
    w[q + ("q" if mixer == "delta" else "r")] = every
    w[q + "k"] = every if mixer == "delta" else ((first + 0.001 * others) * ramp).to(torch.bfloat16)
    if mixer == "delta":   # only token 0 writes
        w[q + "b"], w[q + "a"] = (8.0 * first - 12.0 * others)[None].to(torch.bfloat16), torch.zeros(1, W, dtype=torch.bfloat16)
        w[q + "dt_bias"] = torch.full((1,), -30.0, dtype=torch.bfloat16)
    else:                  # only token 0 has a key that counts; no mixing with the predecessor
        w[q + "w0"] = torch.full((N,), -30.0, dtype=torch.bfloat16)
        w[q + "w2"].zero_(), w[q + "u"].fill_(0.001)
        for s in "rkvgw":
            w[q + "mu." + s].zero_()
    wn = lu.as_numpy(w)
    m = build(cfg, w, dtype)
    for at in (0, 15, 16, 63, 64):
        ids = np.random.default_rng(at).integers(1, V, 300).astype(np.int32)
        ids[at] = 0
        want = orc.forward(cfg, wn, ids)
        other = ids.copy()
        other[at] = 1
        assert lu.err(orc.forward(cfg, wn, other)[200:], want[200:]) > 0.1      # it is remembered
        assert lu.err(whole(m, ids)[at:], want[at:]) < TOL[dtype], at
        assert lu.err(in_portions(m, ids, [40, 42, 130, 145, 146, 290, 291, 292])[at:], want[at:]) < TOL[dtype], at


# ------------------------------------------------------------------ attention
@BOTH
@pytest.mark.parametrize("size", [(3, 3, 8), (4, 2, 17), (6, 2, 32), (2, 1, 50), (4, 4, 64), (3, 1, 96), (2, 2, 130), (2, 1, 200), (1, 1, 256), (2, 1, 300)], ids=str)
def test_every_attention_size_class(size, dtype):
    """(heads, kv_heads, dim): prompts, portions behind them, decoded tokens; heads too wide for the matrix cores."""
    H, G, D = size
    cfg = lu.config([(lu.parallel(lu.left(H, G, D, chunk=170), lu.right(1, 8)), None)])
    w = lu.only(lu.weights(cfg, seed=5, q_gain=2.0), ["left"])
    both_ways(cfg, w, dtype, 330, [180, 325, 328, 329])


@pytest.mark.parametrize("heads", [(1, 1), (31, 1), (33, 33), (48, 3), (130, 2)], ids=str)
def test_every_number_of_heads(heads):
    cfg = lu.config([(lu.parallel(lu.left(*heads, 8, chunk=None), lu.right(1, 8)), None)])
    w = lu.only(lu.weights(cfg, seed=6, q_gain=2.0), ["left"])
    both_ways(cfg, w, torch.bfloat16, 300, [200, 250, 256, 297, 298, 299])


@BOTH
@pytest.mark.parametrize("table", [(2, 3), (7, 20), (12, 12), (16, 130), (32, 250), (64, 2000)], ids=str)
def test_distance_tables(table, dtype):
    """(rows, far): one row of the table outweighs the others, so a distance that is one bucket off shows; tables larger than a workgroup's scratch memory."""
    rows, far = table
    cfg = lu.config([(lu.parallel(lu.left(6, 2, 16, bias_max=far, chunk=None), lu.right(1, 8)), None)], width=64)
    for row in sorted({0, 1, rows // 2, rows - 1}):
        w = lu.only(lu.weights(cfg, seed=11, rel_rows=rows), ["left"])
        w["l0.mix.left.rel"][row] += 5.0
        ids = lu.tokens(cfg, 300)
        wn = lu.as_numpy(w)
        want = orc.forward(cfg, wn, ids)
        m = build(cfg, w, dtype)
        assert lu.err(whole(m, ids), want) < TOL[dtype], row
        assert lu.err(in_portions(m, ids, [130, 132, 290, 291, 292]), want) < TOL[dtype], row


@BOTH
@pytest.mark.parametrize("chunk", [1, 2, 31, 32, 33, 63, 64, 65, 100, 128, 1000])
def test_chunks_of_every_size(chunk, dtype):
    """Chunks that end inside, at and behind pages and key blocks; portions that end inside, at and behind chunks."""
    cfg = lu.config([(lu.parallel(lu.left(4, 2, 16, chunk=chunk), lu.right(1, 8)), None)], width=64)
    w = lu.only(lu.weights(cfg, seed=12, q_gain=2.0), ["left"])
    both_ways(cfg, w, dtype, 270, sorted({max(chunk - 1, 1), chunk + 1, chunk + 2, 2 * chunk + 1, 2 * chunk + 3, 150, 200, 201, 202, 255, 256, 257} & set(range(1, 270))))


def lone_token_keys(w, p, cfg, mx):
    """Attention weights under which token 0's key outscores every other for every query, and its value differs from all others'."""
    W, H, G, D = cfg["width"], mx["heads"], mx["kv_heads"], mx["dim"]
    back = token_projection(w, W)
    k, q = torch.zeros(G, D, W), torch.zeros(H, D, W)
    k[:, 0], k[:, 1] = 3 * back[:, 0], 3 * back[:, 1:].sum(1)
    q[:, 0] = back.sum(1)
    w[p + "k"], w[p + "q"] = k.flatten(0, 1).to(torch.bfloat16), q.flatten(0, 1).to(torch.bfloat16)
    for n in ("k.b", "q.b", "rel", "sink"):
        w[p + n].zero_()
    w[p + "q.norm"].fill_(1.0), w[p + "k.norm"].fill_(1.0)


@BOTH
def test_far_keys(dtype):
    """One token's key outscores every other for every query and decides the output as long as it is seen: at page, block and chunk borders, from its own position to the last
    of its chunk, not one further; in prompts and in decoding."""
    n, chunk = 300, 130
    cfg = lu.config([(lu.parallel(lu.left(2, 1, 16, scale=0.6, chunk=chunk), lu.right(1, 8)), None)], width=64, vocab=50, eps=1e-6)
    w = lu.only(lu.weights(cfg, seed=9), ["left"])
    lone_token_keys(w, "l0.mix.left.", cfg, cfg["layers"][0]["mixer"]["left"])
    wn, m = lu.as_numpy(w), build(cfg, w, dtype)
    for at in (0, 1, 31, 32, 63, 64, 127, 128, 129, 130, 131, 191, 259, 260):
        ids = np.random.default_rng(at).integers(1, 50, n).astype(np.int32)
        ids[at] = 0
        want = orc.forward(cfg, wn, ids)
        other = ids.copy()
        other[at] = 1
        moved, end = np.array([lu.err(a[None], b[None]) for a, b in zip(orc.forward(cfg, wn, other), want)]), min((at // chunk + 1) * chunk, n)
        assert (moved[at:end] > 0.05).all() and (moved[:at] < 1e-9).all() and (moved[end:] < 1e-9).all()   # it decides inside its chunk, and nowhere else
        assert lu.err(whole(m, ids), want) < TOL[dtype], at
        cuts = sorted({*range(at - 2, at + 3), 129, 130, 131, 259, 260, 261, 295, 296, 297, 298, 299} & set(range(1, n)))
        assert lu.err(in_portions(m, ids, cuts), want) < TOL[dtype], at


@BOTH
@pytest.mark.parametrize("level", [-30.0, -2.0, 3.0, 60.0])
def test_the_sinks_count(level, dtype):
    """Sinks far below, around and far above the scores: they decide how large the heads are against each other, at the first tokens of a sequence and of a chunk, in prompts and in decoding."""
    cfg = lu.config([(lu.parallel(lu.left(heads=4, kv_heads=2), lu.right(1, 8)), None)], width=64)
    w = lu.only(lu.weights(cfg, seed=10), ["left"])
    w["l0.mix.left.sink"] = torch.tensor([level, 0.0, -1.0, 2.0], dtype=torch.bfloat16)
    wn, ids = lu.as_numpy(w), lu.tokens(cfg, 200)
    want = orc.forward(cfg, wn, ids)
    without = orc.forward(cfg, wn | {"l0.mix.left.sink": np.full(4, -1e30)}, ids)
    assert min(lu.err(without[i:i + 1], want[i:i + 1]) for i in (0, 1, 5, 70, 140)) > 0.02
    m = build(cfg, w, dtype)
    assert lu.err(whole(m, ids), want) < TOL[dtype] and lu.err(in_portions(m, ids, [1, 2, 3, 100, 140, 141, 198, 199]), want) < TOL[dtype]


@BOTH
def test_scores_far_below_the_sink(dtype):
    """Scores around -150 beside a sink of 5: nothing overflows, and the heads give nothing."""
    cfg = lu.config([(lu.parallel(lu.left(heads=2, kv_heads=1), lu.right(1, 8)), None)], width=64)
    w = lu.only(lu.weights(cfg, seed=10, sink=5.0), ["left"])
    w["l0.mix.left.rel"] -= 150.0
    both_ways(cfg, w, dtype, 150, [1, 2, 90, 148, 149])


# ------------------------------------------------------------------ what surrounds the sublayers
@BOTH
@pytest.mark.parametrize("ff", [1, 8, 13, 130, 700])
def test_every_feed_forward_width(ff, dtype):
    cfg = lu.config([(lu.delta(heads=1, dim=8, vdim=8), lu.dense(ff))], width=76)
    both_ways(cfg, lu.weights(cfg, seed=12), dtype, 100, [60, 97, 98, 99])


@BOTH
@pytest.mark.parametrize("side", [1, 5, 8, 64, 100, 192])
def test_every_side_input_width(side, dtype):
    if side == 1 and dtype == torch.bfloat16:
        pytest.skip("the norm of a multiple of one vector is its sign: near zero, rounding decides it")
    cfg = lu.config([(lu.delta(heads=1, dim=8, vdim=8), None), (lu.delta(heads=1, dim=8, vdim=8), lu.dense(24))], width=76, side=side)
    w = lu.weights(cfg, seed=13)
    for i in range(2):
        w[f"l{i}.side.norm"] *= 3
    both_ways(cfg, w, dtype, 100, [60, 97, 98, 99])


@BOTH
@pytest.mark.parametrize("width", [5, 20, 50, 260, 300, 1028, 2052, 4100])
def test_every_width(width, dtype):
    cfg = lu.config([(lu.parallel(lu.left(2, 1, 8), lu.right(1, 8)), lu.dense(24)), (lu.parallel(lu.left(2, 1, 8), lu.right(1, 8)), None)], width=width, vocab=40, positions=90)
    both_ways(cfg, lu.weights(cfg, seed=12), dtype, 80, [70, 75, 76])


@BOTH
@pytest.mark.parametrize("constants", [(0.3, 0.5), (5.0, 30.0)], ids=str)
def test_constants_come_from_the_configuration(constants, dtype):
    cfg = lu.config([(lu.parallel(scales=(2.5, 0.1)), lu.dense()), (lu.delta(), None)], alpha=constants[0], cap=constants[1], eps=0.1)
    both_ways(cfg, lu.weights(cfg, seed=14), dtype, 90, [70, 85, 86])


# ------------------------------------------------------------------ the whole model
@BOTH
def test_wider_layers_and_longer_prompts(dtype):
    """Several row and column tiles everywhere, and one pass of long and short runs together."""
    cfg = lu.config([(lu.parallel(lu.left(8, 4, 64, chunk=300), lu.right(6, 64)), lu.dense(700)), (lu.delta(6, 3, 64, 96, 4), None), (lu.parallel(lu.left(4, 1, 128, chunk=None, bias_max=500), lu.right(3, 96)), None)],
                    width=328, vocab=600, positions=800, side=72)
    w = lu.weights(cfg, seed=17)
    m, wn = build(cfg, w, dtype), lu.as_numpy(w)
    todo = [lu.sequence(cfg, wn, n, seed=n) for n in (700, 5, 130, 66, 1, 63)]
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
            assert lu.err(got[at:at + len(r)], r) < TOL[dtype], len(r)
            at += len(r)


def test_long_prompts_take_several_segments(monkeypatch):
    """More chunks than one segment of a scan's operands holds, over several runs."""
    cfg = lu.config([(lu.delta(16, 16, 128, 128), None), (lu.parallel(lu.left(2, 1, 16), lu.right(16, 128)), None)], width=64, vocab=60, positions=2600)
    w = lu.weights(cfg, seed=19)
    wn, m = lu.as_numpy(w), build(cfg, w, torch.bfloat16, pages=80)
    todo = [lu.sequence(cfg, wn, n, seed=n) for n in (2500, 700, 40)]
    got = m.step_portions([(t, m.make_cache()) for t, _ in todo], [list(range(len(t))) for t, _ in todo]).cpu().numpy()
    at = 0
    for t, want in todo:
        assert lu.err(got[at:at + len(t)], want) < TOL[torch.bfloat16], len(t)
        at += len(t)


@BOTH
def test_prompt_equals_token_by_token(dtype):
    cfg = lu.CONFIGS["mixed"]
    w = lu.weights(cfg, seed=6, q_gain=1.5)
    m = build(cfg, w, dtype)
    ids, want = lu.sequence(cfg, lu.as_numpy(w), 135)
    c = m.make_cache()
    got = []
    for t in ids:
        _, _, logits = m.step(torch.tensor([t], dtype=torch.int32), c)   # captured and replayed from the third step on
        got.append(logits.cpu().numpy().copy())
    assert lu.err(np.stack(got), want) < TOL[dtype]


@BOTH
@pytest.mark.parametrize("cut", [2, 3, 7, 16, 31, 64, 65, 100])
def test_portions(cut, dtype):
    cfg = lu.CONFIGS["mixed"]
    w = lu.weights(cfg, seed=21, q_gain=1.5)
    ids, want = lu.sequence(cfg, lu.as_numpy(w), 203)
    assert lu.err(in_portions(build(cfg, w, dtype), ids, list(range(cut, 203, cut))), want) < TOL[dtype]


@BOTH
def test_mixed_batches_reuse_pages_and_slots(dtype):
    """Unequal requests side by side -- portions, single tokens, requests left out of a step -- in a pool so small that pages and slots come back."""
    cfg = lu.CONFIGS["mixed"]
    w, rng = lu.weights(cfg, seed=8, q_gain=1.5), np.random.default_rng(0)
    m, wn = build(cfg, w, dtype, pages=9, slots=4), lu.as_numpy(w)
    todo = [lu.sequence(cfg, wn, int(n), seed=100 + i) for i, n in enumerate((130, 70, 5, 65, 128, 1, 90, 33, 64, 127))]
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
            assert lu.err(got[at:at + n], todo[i][1][lo:lo + n]) < TOL[dtype], (i, lo, n)
            at += n
            live[i][1] = lo + n
            used.update(live[i][0][0].page_manager.pages)
            slots.add(live[i][0][0].page_manager.slot)
            if lo + n == len(todo[i][0]):
                live.pop(i)[0][0].page_manager.release()
    assert m._pool.get_num_free_pages() == 9 and m._pool.num_free_slots() == 4 and len(used) <= 9 and slots <= set(range(4))


@BOTH
def test_long_decoding(dtype):
    cfg = lu.CONFIGS["mixed"]
    w = lu.weights(cfg, seed=10, q_gain=1.5)
    m = build(cfg, w, dtype)
    ids, want = lu.sequence(cfg, lu.as_numpy(w), 500)
    c = m.make_cache()
    m.step_portions([(ids[:20], c)], [[]])
    got = []
    for t in ids[20:]:
        got.append(m.step_batch(torch.tensor([t]), [c])[2].clone())
    assert lu.err(torch.cat(got).cpu().numpy(), want[20:]) < TOL[dtype]


@BOTH
@pytest.mark.parametrize("batch", [5, 20, 40, 70])
def test_batches_of_decoded_tokens(batch, dtype):
    """Every row count class of the few-row kernels, and the many-row ones, with single rows only."""
    cfg = lu.CONFIGS["mixed"]
    w = lu.weights(cfg, seed=11)
    m, wn = build(cfg, w, dtype, pages=batch * 2, slots=batch), lu.as_numpy(w)
    todo = [lu.sequence(cfg, wn, 20 + i % 50, seed=i) for i in range(batch)]
    caches = [m.make_cache() for _ in todo]
    m.step_portions([(t[:-4], c) for (t, _), c in zip(todo, caches)], [[]] * batch)
    for k in range(4, 0, -1):
        got = m.step_batch(torch.tensor([t[-k] for t, _ in todo]), caches)[2].cpu().numpy()
        assert lu.err(got, np.stack([want[-k] for _, want in todo])) < TOL[dtype]


@BOTH
@pytest.mark.parametrize("size", [(128, 128), (96, 256), (40, 100)], ids=str)
def test_many_states_at_once(size, dtype):
    """More (sequence, head) pairs than compute units, decoded and in short portions: wide heads take other workgroup shapes then."""
    D, V = size
    cfg = lu.config([(lu.delta(8, 4, D, V, 4), None), (lu.parallel(lu.left(2, 1, 8), lu.right(8, D)), None)], width=64, vocab=60)
    w = lu.weights(cfg, seed=20)
    m, wn = build(cfg, w, dtype, pages=50, slots=42), lu.as_numpy(w)
    todo = [lu.sequence(cfg, wn, 12 + i % 9, seed=i) for i in range(42)]
    caches = [m.make_cache() for _ in todo]
    m.step_portions([(t[:-6], c) for (t, _), c in zip(todo, caches)], [[]] * 42)
    got = m.step_portions([(t[-6:-3], c) for (t, _), c in zip(todo, caches)], [[0, 1, 2]] * 42).cpu().numpy()
    assert lu.err(got, np.concatenate([want[-6:-3] for _, want in todo])) < TOL[dtype]
    for k in range(3, 0, -1):
        got = m.step_batch(torch.tensor([t[-k] for t, _ in todo]), caches)[2].cpu().numpy()
        assert lu.err(got, np.stack([want[-k] for _, want in todo])) < TOL[dtype], k


def test_logits_do_not_depend_on_the_batch():
    """The same request alone and among 20 others: equal to rounding, far below what bf16 itself costs."""
    cfg = lu.CONFIGS["mixed"]
    w = lu.weights(cfg, seed=11)
    m, wn = build(cfg, w, torch.bfloat16, pages=128), lu.as_numpy(w)
    ids, _ = lu.sequence(cfg, wn, 100)
    alone = whole(m, ids)
    caches = [m.make_cache() for _ in range(21)]
    entries = [(lu.tokens(cfg, 3 + 11 * i, seed=i), caches[i]) for i in range(20)] + [(ids, caches[20])]
    got = m.step_portions(entries, [[] for _ in range(20)] + [list(range(100))]).cpu().numpy()
    assert lu.err(got, alone) < 0.02


def test_graph_replays_equal_launches():
    """A captured step replayed many times, with other work and synchronisation between, against the same step as launches."""
    cfg = lu.CONFIGS["mixed"]
    w = lu.weights(cfg, seed=12)
    m = build(cfg, w, torch.bfloat16)
    prompts = [lu.tokens(cfg, n, seed=n) for n in (30, 64, 7)]
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
    cfg = lu.CONFIGS["mixed"]
    w = lu.weights(cfg, seed=18)
    m, wn = build(cfg, w, torch.float32), lu.as_numpy(w)
    todo = [lu.sequence(cfg, wn, 40, seed=s) for s in (1, 2)]
    caches = [m.make_cache() for _ in todo]
    for t in range(40):
        for (ids, want), c in zip(todo, caches):
            got = m.step_batch(torch.tensor([ids[t]]), [c])[2].cpu().numpy()
            assert lu.err(got, want[t:t + 1]) < 1e-4, t


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
    cfg = lu.CONFIGS["mixed"]
    w = lu.weights(cfg, seed=13)
    wn, m = lu.as_numpy(w), build(cfg, w, torch.float32)
    common = list(lu.tokens(cfg, 70, seed=50))
    prompts = [common + list(lu.tokens(cfg, n, seed=60 + n)) for n in (3, 20, 41, 9, 1)]
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
    cfg = lu.CONFIGS["mixed"]
    m = build(cfg, lu.weights(cfg, seed=14), torch.bfloat16)
    eng = InferenceEngine(model=m)
    eng.prompt_cache = PromptCache(directory=tmp_path)
    prompt = lu.tokens(cfg, 12)
    eng.prepare_engine(prompt, temp=0.8, top_p=0.9, repetition_penalty=1.2)
    out = [t for t, _ in eng.generate(prompt, max_completion_tokens=6)]
    assert len(out) == 6 and all(0 <= t < cfg["vocab"] for t in out)


def test_positions_end():
    """A sequence cannot grow beyond the position vectors: passes are refused, the engine stops."""
    from proxy_inference_engine_amd.engine import BatchedEngine
    cfg = lu.config([(lu.parallel(), None)], width=40, positions=20)
    w = lu.weights(cfg, seed=15)
    wn, m = lu.as_numpy(w), build(cfg, w, torch.float32)
    ids, want = lu.sequence(cfg, wn, 20)
    c = m.make_cache()
    with pytest.raises(ValueError, match="20 positions"):
        m.step_portions([(list(ids) + [1], c)], [[]])
    got = m.step_portions([(ids, c)], [list(range(20))]).cpu().numpy()
    assert lu.err(got, want) < 5e-5
    with pytest.raises(ValueError, match="20 positions"):
        m.step_batch(torch.tensor([1]), [c])
    prompts = [[int(t) for t in ids[:17]], [int(t) for t in ids], [3]]
    expect = [greedy(cfg, wn, p, n) for p, n in zip(prompts, (4, 1, 8))]
    assert BatchedEngine(m, num_pages=4, max_batch=2).generate(prompts, 8) == expect


def test_prompts_longer_than_a_pass(monkeypatch):
    from proxy_inference_engine_amd.models import layer_stack
    cfg = lu.CONFIGS["mixed"]
    w, ids = lu.weights(cfg, seed=15), lu.tokens(cfg, 170)
    m, want = build(cfg, w, torch.float32), orc.forward(cfg, lu.as_numpy(w), ids)
    monkeypatch.setattr(layer_stack, "MAX_ROWS", 50)
    a, b = m.make_cache(), m.make_cache()
    got = m.step_portions([(ids, a), (ids[:90], b)], [[0, 49, 50, 169], [89]]).cpu().numpy()
    assert lu.err(got, want[[0, 49, 50, 169, 89]]) < TOL[torch.float32]


def test_bad_models_and_calls_are_refused():
    cfg = lu.CONFIGS["mixed"]
    w = lu.weights(cfg)
    m = build(cfg, w, torch.bfloat16, pages=3, slots=2)
    a, b, c = (m.make_cache() for _ in range(3))
    with pytest.raises(RuntimeError, match="exhausted"):
        m.step_portions([(lu.tokens(cfg, 200), a)], [[]])
    assert a[0].offset == 0 and m._pool.get_num_free_pages() == 3 and m._pool.num_free_slots() == 2
    m.step_portions([([1, 2], a), ([3], b)], [[], []])
    with pytest.raises(RuntimeError, match="slots"):
        m.step_portions([([1], c)], [[]])
    from proxy_inference_engine_amd.models.lagelorn import Model, ModelArgs
    dev = {k: v.cuda() for k, v in w.items()}
    for change in (lambda d: d["layers"][0]["mixer"]["left"].update(kv_heads=3), lambda d: d["layers"][0]["mixer"]["left"].update(vdim=16), lambda d: d["layers"][1].update(type="other"),
                   lambda d: d["layers"][2]["mixer"].update(kv_heads=3), lambda d: d["layers"][0]["mlp"].update(kind="other"), lambda d: d["layers"][1]["mixer"].update(conv=17),
                   lambda d: d["layers"][0]["mixer"].update(right=None), lambda d: d["token_side"].update(dim=15)):
        bad = json.loads(json.dumps(cfg))
        change(bad)
        with pytest.raises(ValueError):
            Model(ModelArgs(**bad), dev)
    with pytest.raises(ValueError, match="missing"):
        Model(ModelArgs(**cfg), {k: v for k, v in dev.items() if k != "l0.mix.right.w2"})


def test_what_layers_cache():
    cfg = lu.CONFIGS["mixed"]
    m = build(cfg, lu.weights(cfg), torch.bfloat16)
    assert m.row_elems == [2 * (32 + 32), 0, 0, 2 * (16 + 32), 3 * (48 + 64)]
    assert m.state_floats == [3 * 20 * 20 + 112, 3 * 20 * 28 + 3 * (2 * 3 * 24 + 3 * 32), 4 * 16 * 40 + 5 * (2 * 2 * 16 + 4 * 40), 2 * 33 * 33 + 2 + 112, 5 * 7 * 7 + 3 + 112]


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_runner(tmp_path, dtype):
    """bin/trace_run on a checkpoint written to disk: two requests, portions beside single tokens, pages and slots used again."""
    from safetensors.torch import save_file
    cfg = lu.CONFIGS["mixed"]
    w = lu.weights(cfg, seed=16)
    wn = lu.as_numpy(w)
    save_file(w, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    (a, wa), (b, wb) = lu.sequence(cfg, wn, 80, seed=1), lu.sequence(cfg, wn, 66, seed=2)
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
        assert lu.err(got, np.stack(want)) < TOL[getattr(torch, dtype)], i
