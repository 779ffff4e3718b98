"""Kodupel without a GPU: configuration, registry, page and slot bookkeeping, prompt reuse, and the oracle against itself."""
import json

import numpy as np
import pytest
import torch

import kodupel_util as ku
from oracle import kodupel_oracle as orc
from proxy_inference_engine_amd.cache import PromptCache
from proxy_inference_engine_amd.cache.kv_cache import BaseCache, PagedStackCache, SavedStackCache, StackPageAllocator, StackSequence
from proxy_inference_engine_amd.models import utils as mu
from proxy_inference_engine_amd.models.kodupel import ModelArgs
from proxy_inference_engine_amd.models.layer_stack import yarn_frequencies


def test_config_is_read_layer_by_layer():
    a = ModelArgs(**json.loads(json.dumps(ku.CONFIGS["mixed"])))
    assert [lay.type for lay in a.layers] == ["attention", "general_delta", "attention", "attention", "general_delta", "attention"]
    assert [lay.mixer.kv_from for lay in a.layers] == [None, None, None, 0, None, 2] and a.layers[2].mixer.rot.scaling is None
    assert a.layers[0].mixer.rot.scaling.slow == 1.0 and a.layers[1].mlp.expert.limit == 0.7 and a.layers[2].mlp is None and a.embedding.scale == 0.7


def test_registry_knows_the_design():
    assert "Kodupel" in mu._ARCHITECTURES


@pytest.mark.parametrize("dims,base,scaling", [(8, 5000.0, (4.0, 64, 16.0, 1.0)), (24, 1e4, (2.0, 4096, 32.0, 1.0)), (2, 10.0, (8.0, 128, 2.0, 2.0)), (64, 5e5, None),
                                               (16, 100.0, (1.5, 10, 1e-3, 1e-4))], ids=str)
def test_frequencies(dims, base, scaling):
    f, gain = yarn_frequencies(dims, base, scaling)
    want, want_gain = orc.rotary_frequencies(dims, base, None if scaling is None else dict(zip(("factor", "original", "fast", "slow"), scaling)))
    assert np.allclose(f.numpy(), want, rtol=1e-6) and gain == pytest.approx(want_gain) and f.dtype == torch.float32


def pool(pages=4, slots=2, states=(0, 6)):
    return StackPageAllocator(pages, [16, 0], list(states), slots, dtype=torch.float32, device="cpu")


def test_slots_come_and_go_with_the_tokens():
    a = pool()
    seqs = [StackSequence(a, 1) for _ in range(3)]
    assert a.num_free_slots() == 2 and all(s.slot is None for s in seqs)   # nothing is held before the first token
    seqs[0].reserve(1), seqs[0].advance(1), seqs[1].reserve(70), seqs[1].advance(70)
    assert a.num_free_slots() == 0 and seqs[0].slot != seqs[1].slot
    with pytest.raises(RuntimeError, match="slots"):
        seqs[2].reserve(1)
    assert a.get_num_free_pages() == 1 and seqs[2].pages == []
    with pytest.raises(RuntimeError, match="exhausted"):   # pages: nothing is left behind
        seqs[0].reserve(200)
    assert seqs[0].slot is not None
    held = seqs[0].slot
    seqs[0].release()
    seqs[2].reserve(1)
    assert seqs[2].slot == held
    with pytest.raises(ValueError):
        seqs[1].truncate(10)                               # a recurrent state cannot go back
    seqs[1].truncate(70)
    assert seqs[1].offset == 70 and seqs[1].keepable(70) == 70 and seqs[1].keepable(69) == 0
    seqs[1].release(), seqs[2].release()
    assert a.num_free_slots() == 2 and a.get_num_free_pages() == 4


def test_a_failed_first_reservation_keeps_no_slot():
    a = pool(pages=1)
    s = StackSequence(a, 1)
    with pytest.raises(RuntimeError, match="exhausted"):
        s.reserve(100)
    assert s.slot is None and a.num_free_slots() == 2 and a.get_num_free_pages() == 1


def test_without_recurrent_layers_there_are_no_slots():
    a = pool(states=(0, 0), slots=1)
    s, t = StackSequence(a, 1), StackSequence(a, 1)
    s.reserve(70), s.advance(70), t.reserve(1)
    assert s.slot is None and s.keepable(10) == 10
    s.truncate(10)
    assert s.offset == 10 and len(s.pages) == 1


def test_fork_copies_the_state():
    a = pool()
    s = StackSequence(a, 1)
    s.reserve(64), s.advance(64)
    a.states[1][s.slot] = torch.arange(6.0)
    t = s.fork()
    assert t.slot not in (None, s.slot) and torch.equal(a.states[1][t.slot], torch.arange(6.0)) and t.pages == s.pages and t.offset == 64
    with pytest.raises(RuntimeError):
        s.fork()
    s.release()
    assert a.get_num_free_pages() == 3                     # the page is still the other's
    t.release()
    assert a.get_num_free_pages() == 4 and a.num_free_slots() == 2


def test_saved_pages_and_state_round_trip(tmp_path):
    a = pool(pages=8)
    seq = StackSequence(a, 2)
    seq.reserve(70), seq.advance(70)
    a.slabs[0].copy_(torch.randn_like(a.slabs[0]))
    a.states[1][seq.slot] = torch.randn(6)
    cache = [PagedStackCache(seq, i) for i in range(2)]
    BaseCache.save_cache(str(tmp_path / "c.safetensors"), cache, {"k": "v"})
    back, meta = BaseCache.load_cache(str(tmp_path / "c.safetensors"), device="cpu")
    assert all(isinstance(c, SavedStackCache) and c.offset == 70 for c in back) and meta == {"k": "v"}
    other = StackSequence(a, 2)
    mine = [PagedStackCache(other, i) for i in range(2)]
    for m, saved in zip(mine, back):
        m.adopt(saved)
    assert other.offset == 70 and other.slot != seq.slot and torch.equal(a.states[1][other.slot], a.states[1][seq.slot])
    assert all(torch.equal(a.slabs[0][p], a.slabs[0][q]) for p, q in zip(seq.pages, other.pages))


@pytest.mark.parametrize("states,kept", [((0, 6), (70, 0)), ((0, 0), (70, 40))], ids=["recurrent", "attention_only"])
def test_prompt_reuse(states, kept, tmp_path):
    """All of the history is kept, or -- where a state would have to go back -- none of it; without recurrent layers the common prefix."""
    for common, expect in zip((70, 40), kept):
        a = pool(pages=4, states=states)
        seq = StackSequence(a, 2)
        seq.reserve(70), seq.advance(70)
        history = list(range(70))
        pc = PromptCache(directory=tmp_path, cache=[PagedStackCache(seq, i) for i in range(2)], computed_ids=history)
        prompt = history[:common] + [500, 501, 502]
        assert pc.reuse_cache(prompt) == prompt[expect:] and pc.computed_ids == history[:expect] and seq.offset == expect
        assert (seq.slot is None) == (expect == 0 or not any(states))


# ------------------------------------------------------------------ the oracle against itself
def test_oracle_recurrence_continues_from_its_state():
    rng = np.random.default_rng(0)
    r, k, v = (rng.normal(size=(11, 2, 5)) for _ in range(3))
    w, a = 0.5 + 0.5 * rng.random((11, 2, 5)), rng.random((11, 2, 5))
    whole, end = orc.delta_recurrence(r, k, v, w, a)
    first, state = orc.delta_recurrence(r[:4], k[:4], v[:4], w[:4], a[:4])
    rest, end2 = orc.delta_recurrence(r[4:], k[4:], v[4:], w[4:], a[4:], state)
    assert np.allclose(np.concatenate([first, rest]), whole) and np.allclose(end, end2)


def test_oracle_rotation_is_relative():
    f, gain = orc.rotary_frequencies(8, 100.0, {"factor": 2.0, "original": 32, "fast": 4.0, "slow": 1.0})
    rng = np.random.default_rng(1)
    q, k = rng.normal(size=(1, 1, 12)), rng.normal(size=(1, 1, 12))

    def score(i, j):
        return float((orc.rotate_pairs(q, np.array([float(i)]), f, gain) * orc.rotate_pairs(k, np.array([float(j)]), f, gain)).sum())
    assert score(9, 4) == pytest.approx(score(105, 100)) and abs(score(9, 4) - score(9, 5)) > 1e-3


MISTAKES = ["sink", "scale", "gate", "q_norm", "k_norm", "v_norm", "rotation", "interleave", "yarn_gain", "yarn_freq", "q_bias", "o_bias", "group", "kv_from", "decay", "removal",
            "unit_key", "old_state", "head_norm", "delta_gate", "rate_bias", "state_lost", "limit", "slope", "up_one", "correction", "weight_correction", "top",
            "zero_centred", "embed_scale"]


@pytest.mark.parametrize("mistake", MISTAKES)
def test_oracle_mistakes_show(mistake, monkeypatch):
    """With weights like those of the device tests, every mechanism left out or replaced moves the logits: by a thousand times what the
    32-bit tests allow at least."""
    cfg = json.loads(json.dumps(ku.CONFIGS["mixed"]))
    w, ids = ku.as_numpy(ku.weights(cfg, seed=3, q_gain=1.5)), ku.tokens(cfg, 80)
    want = orc.forward(cfg, w, ids)

    def without_norm(which):
        for name in w:
            if name.endswith(which):
                w[name] = np.ones_like(w[name])
    real = {n: getattr(orc, n) for n in ("sink_softmax", "unit_rms", "rotate_pairs", "rotary_frequencies", "delta_recurrence", "choose_experts", "keys_values", "clipped_expert", "sigmoid",
                                         "attention", "general_delta", "delta_decay")}
    patch = lambda name, f: monkeypatch.setattr(orc, name, f)  # noqa: E731

    def plain_softmax(s, mask):
        s = np.where(mask, s, -np.inf)
        p = np.exp(s - s.max(-1, keepdims=True))
        return p / p.sum(-1, keepdims=True)

    def recurrence(change):
        return lambda r, k, v, d, a, state=None: real["delta_recurrence"](*change(r, k, v, d, a))
    if mistake == "sink":
        patch("sink_softmax", plain_softmax)
    elif mistake == "scale":
        cfg["layers"][5]["mixer"]["scale"] = 40 ** -0.5
    elif mistake == "gate":
        for n in [n for n in w if n.endswith("mix.g") and w[n].shape[0] < 20 and "l1" not in n and "l4" not in n]:
            w[n] = np.zeros_like(w[n])
    elif mistake in ("q_norm", "k_norm"):
        without_norm("." + mistake.replace("_", "."))
    elif mistake == "v_norm":
        def kv(h, w, p, mx, eps):
            k, _ = real["keys_values"](h, w, p, mx, eps)
            return k, (h @ w[p + "v"].T + w[p + "v.b"]).reshape(len(h), mx["kv_heads"], mx["vdim"])
        patch("keys_values", kv)
    elif mistake == "rotation":
        patch("rotate_pairs", lambda x, pos, f, g: x)
    elif mistake == "interleave":
        def halves(x, pos, f, g):
            n = len(f)
            y = x.copy()
            y[..., 0:2 * n:2], y[..., 1:2 * n:2] = x[..., :n], x[..., n:2 * n]
            y = real["rotate_pairs"](y, pos, f, g)
            z = y.copy()
            z[..., :n], z[..., n:2 * n] = y[..., 0:2 * n:2], y[..., 1:2 * n:2]
            return z
        patch("rotate_pairs", halves)
    elif mistake == "yarn_gain":
        patch("rotary_frequencies", lambda d, b, s=None: (real["rotary_frequencies"](d, b, s)[0], 1.0))
    elif mistake == "yarn_freq":
        patch("rotary_frequencies", lambda d, b, s=None: (real["rotary_frequencies"](d, b)[0], real["rotary_frequencies"](d, b, s)[1]))
    elif mistake in ("q_bias", "o_bias"):
        for n in [n for n in w if n.endswith("mix." + mistake[0] + ".b")]:
            w[n] = np.zeros_like(w[n])
    elif mistake == "group":
        def kv(h, w, p, mx, eps):
            k, v = real["keys_values"](h, w, p, mx, eps)
            return k[:, ::-1], v[:, ::-1]
        patch("keys_values", kv)
    elif mistake == "kv_from":
        del cfg["layers"][5]["mixer"]["kv_from"]            # the layer's own input through the other layer's projections
        w |= {"l5." + n[3:]: t for n, t in w.items() if n.startswith("l2.mix.k") or n.startswith("l2.mix.v")}
    elif mistake == "decay":
        patch("delta_decay", lambda h, w, p: np.exp(-orc.sigmoid(np.tanh(h @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"])))
    elif mistake == "removal":
        patch("delta_recurrence", recurrence(lambda r, k, v, d, a: (r, k, v, d, 0 * a)))
    elif mistake == "unit_key":
        patch("delta_recurrence", recurrence(lambda r, k, v, d, a: (r, k / np.linalg.norm(k, axis=-1, keepdims=True), v, d, a)))
    elif mistake == "old_state":   # the removal reads the decayed state
        def after(r, k, v, d, a, state=None):
            S, o, u = np.zeros((r.shape[1], r.shape[2], r.shape[2])), np.empty_like(r), k / np.sqrt(np.sum(k * k, -1, keepdims=True) + 1e-6)
            for t in range(len(r)):
                S = d[t][:, :, None] * S
                S = S - (a[t] * u[t])[:, :, None] * np.einsum("hd,hde->he", u[t], S)[:, None, :] + k[t][:, :, None] * v[t][:, None, :]
                o[t] = np.einsum("hde,hd->he", S, r[t])
            return o, S
        patch("delta_recurrence", after)
    elif mistake == "head_norm":
        without_norm("mix.norm")
    elif mistake == "delta_gate":
        for n in ("l1.mix.g", "l4.mix.g"):
            w[n] = np.zeros_like(w[n])
    elif mistake == "rate_bias":
        for n in ("l1.mix.a.b", "l4.mix.a.b"):
            w[n] = np.zeros_like(w[n])
    elif mistake == "state_lost":
        def lose(r, k, v, d, a, state=None):
            parts = [real["delta_recurrence"](r[i:i + 40], k[i:i + 40], v[i:i + 40], d[i:i + 40], a[i:i + 40])[0] for i in range(0, len(r), 40)]
            return np.concatenate(parts), None
        patch("delta_recurrence", lose)
    elif mistake == "limit":
        for lay in cfg["layers"]:
            if lay["mlp"]:
                lay["mlp"]["expert"]["limit"] = 1e9
    elif mistake in ("slope", "up_one"):
        slope, one = (1.0, 1.0) if mistake == "slope" else (1.702, 0.0)

        def expert(h, w, p, limit):
            g, u = np.minimum(h @ w[p + "gate"].T, limit), np.clip(h @ w[p + "up"].T, -limit, limit)
            return (g * orc.sigmoid(slope * g) * (u + one)) @ w[p + "down"].T
        patch("clipped_expert", expert)
    elif mistake == "correction":
        for n in [n for n in w if n.endswith("correction")]:
            w[n] = np.zeros_like(w[n])
    elif mistake == "weight_correction":   # (a factor common to a token's experts is lost in the norm behind them: renormalising is not seen)
        def choose(h, w, p, top):
            best, weight, lead = real["choose_experts"](h, w, p, top)
            return best, weight + w[p + "correction"][best], lead
        patch("choose_experts", choose)
    elif mistake == "top":
        cfg["layers"][0]["mlp"]["router"]["top"] = 1
    elif mistake == "zero_centred":
        patch("zero_centred_norm", lambda x, w, eps: orc.unit_rms(x, eps) * w)
    elif mistake == "embed_scale":
        cfg["embedding"]["scale"] = 1.0
    moved = ku.err(orc.forward(cfg, w, ids), want)
    assert moved > 0.03, moved
