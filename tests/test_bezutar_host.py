"""Bezutar without a GPU: configuration, registry, lengths, and the oracle against itself."""
import json

import numpy as np
import pytest

import bezutar_util as bu
from oracle import bezutar_oracle as orc
from proxy_inference_engine_amd.models import utils as mu
from proxy_inference_engine_amd.models.bezutar import ModelArgs


def test_config_is_read_layer_by_layer():
    a = ModelArgs(**json.loads(json.dumps(bu.CONFIGS["mixed"])))
    assert [lay.type for lay in a.layers] == [m[0] for m, _ in bu.MIXED]
    assert [lay.mixer.kv_from for lay in a.layers] == [None, None, None, 0, None, None, None, 5] and a.layers[5].mixer.rot.scaling is None
    assert a.layers[0].mixer.rot.scaling.slow == 1.0 and a.layers[4].mixer.gate_cap == 4.0 and a.layers[6].mixer.width == 50 and a.layers[3].mlp is None
    assert (a.streams, a.canon.taps, a.max_positions) == (3, 5, 600) and (a.embedding.bigram.buckets, a.embedding.bigram.mul_prev, a.embedding.bigram.mul_cur) == (97, 31, 5)


def test_registry_knows_the_design():
    assert "Bezutar" in mu._ARCHITECTURES


# ------------------------------------------------------------------ the oracle against itself
def test_oracle_recurrences_continue_from_their_states():
    rng = np.random.default_rng(0)
    q, k, v = rng.normal(size=(11, 2, 5)), rng.normal(size=(11, 2, 5)), rng.normal(size=(11, 2, 3))
    i, f = rng.normal(size=(11, 2)), -rng.random((11, 2))
    whole, end = orc.mlstm_recurrence(q, k, v, i, f)
    first, state = orc.mlstm_recurrence(q[:4], k[:4], v[:4], i[:4], f[:4])
    rest, end2 = orc.mlstm_recurrence(q[4:], k[4:], v[4:], i[4:], f[4:], state)
    assert np.allclose(np.concatenate([first, rest]), whole) and all(np.allclose(a, b) for a, b in zip(end, end2))
    z, u = rng.random((11, 6)), rng.normal(size=(11, 6))
    whole, end = orc.mingru_recurrence(z, u)
    first, state = orc.mingru_recurrence(z[:4], u[:4])
    rest, end2 = orc.mingru_recurrence(z[4:], u[4:], state)
    assert np.allclose(np.concatenate([first, rest]), whole) and np.allclose(end, end2)


def test_oracle_memory_is_a_sum_over_the_past():
    """The running maximum cancels (but for the floor and the epsilon below the line): sums over earlier tokens with plain products of the gates."""
    rng = np.random.default_rng(1)
    q, k, v = rng.normal(size=(7, 1, 4)), rng.normal(size=(7, 1, 4)), rng.normal(size=(7, 1, 2))
    i, f = rng.normal(size=(7, 1)) + 3, -rng.random((7, 1))
    o, _ = orc.mlstm_recurrence(q, k, v, i, f)
    t = 6
    w = np.array([np.exp(f[s + 1:t + 1].sum() + i[s, 0]) * (k[s, 0] @ q[t, 0]) for s in range(7)])
    assert np.allclose(o[t, 0], w @ v[:, 0] / max(abs(w.sum()), 1.0), rtol=1e-4)


def test_oracle_rotation_is_relative():
    r = {"dims": 8, "base": 100.0, "scaling": {"factor": 2.0, "original": 32, "fast": 4.0, "slow": 1.0}}
    rng = np.random.default_rng(1)
    q, k = rng.normal(size=(1, 1, 12)), rng.normal(size=(1, 1, 12))

    def score(i, j):
        return float((orc.rotate_halves(q, np.array([float(i)]), r) * orc.rotate_halves(k, np.array([float(j)]), r)).sum())
    assert score(9, 4) == pytest.approx(score(105, 100)) and abs(score(9, 4) - score(9, 5)) > 1e-3


def test_oracle_convolution_is_causal():
    h, w = np.zeros((6, 2)), np.array([[1.0, 2.0, 3.0], [0.0, 0.0, 0.5]])
    h[2] = 1.0
    assert orc.causal_conv(h, w).tolist() == [[0, 0], [0, 0], [4, 1.5], [2, 0], [1, 0], [0, 0]]


def test_oracle_bigrams():
    assert orc.bigram_rows([5, 6, 5], 10, 3, 4) == [10, (15 + 24) % 10, (18 + 20) % 10]


MISTAKES = ["sink", "sink_scaled", "scale", "gate", "q_norm", "c_norm", "rotation", "neighbours", "rotated_key_normed", "yarn_gain", "yarn_freq", "kv_from", "shared_own_rank", "floor", "input_cap", "forget_gate", "forget_cap", "key_scale", "mlstm_norm", "mlstm_gate", "state_lost", "candidate", "gru_state_lost", "gru_gate", "gru_bias", "conv", "conv_order",
            "conv_lost", "conv_alone", "streams_in", "streams_transposed", "streams_out", "bigram", "bigram_first", "bigram_order", "positions", "xielu_up", "xielu_down",
            "xielu_slope", "zero_centred"]


@pytest.mark.parametrize("mistake", MISTAKES)
def test_oracle_mistakes_show(mistake, monkeypatch):
    """With weights like those of the device tests, every mechanism left out or replaced moves the logits: by several hundred times what the 32-bit tests allow."""
    cfg = json.loads(json.dumps(bu.CONFIGS["mixed"]))
    if mistake in ("floor", "key_scale"):   # (the head's norm takes any factor out again, unless its epsilon counts)
        cfg["norm"]["eps"] = 0.3
    w, ids = bu.as_numpy(bu.weights(cfg, seed=3, q_gain=1.5, entry=-2.0 if mistake in ("floor", "key_scale") else 0.0)), bu.tokens(cfg, 80)
    want = orc.forward(cfg, w, ids)
    real = {n: getattr(orc, n) for n in ("sink_softmax", "rotate_halves", "rotary_frequencies", "latents", "mlstm_recurrence", "mingru_recurrence", "causal_conv", "streams_in", "streams_out",
                                         "bigram_rows", "xielu", "capped", "softplus")}
    patch = lambda name, f: monkeypatch.setattr(orc, name, f)  # noqa: E731

    def change(end, f=np.zeros_like):
        found = [n for n in w if n.endswith(end)]
        assert found
        for n in found:
            w[n] = f(w[n])

    def memory(cap_i=lambda i: i, cap_f=lambda f: f, floor=True, key=1.0):
        def run(q, k, v, i, f, state=None):
            i, f = cap_i(i), cap_f(f)
            S, z, m, o = np.zeros(k.shape[1:] + v.shape[2:]), np.zeros(k.shape[1:]), np.zeros(k.shape[1]), np.empty_like(v)
            for t in range(len(q)):
                new = np.maximum(f[t] + m, i[t])
                a, b = np.exp(f[t] + m - new), np.exp(i[t] - new)
                S, z, m = a[:, None, None] * S + key * b[:, None, None] * k[t][:, :, None] * v[t][:, None], a[:, None] * z + key * b[:, None] * k[t], new
                nq = np.abs((z * q[t]).sum(1))
                o[t] = np.einsum("hde,hd->he", S, q[t]) / ((np.maximum(nq, np.exp(-m)) if floor else nq) + 1e-6)[:, None]
            return o, None
        patch("mlstm_recurrence", run)

    def cut(f, *args):
        return np.concatenate([f(*(a[i:i + 40] for a in args))[0] for i in range(0, len(args[0]), 40)]), None

    if mistake == "sink":
        patch("sink_softmax", lambda s, mask, sink: real["sink_softmax"](s, mask, -1e30))
    elif mistake == "sink_scaled":
        patch("sink_softmax", lambda s, mask, sink: real["sink_softmax"](s, mask, 0.2 * sink))
    elif mistake == "scale":
        cfg["layers"][3]["mixer"]["scale"] = 20 ** -0.5
    elif mistake == "gate":
        for i in (0, 3, 5, 7):
            change(f"l{i}.mix.g")
    elif mistake in ("q_norm", "c_norm"):
        change("dq.norm" if mistake[0] == "q" else "dkv.norm", np.ones_like)
    elif mistake == "rotation":
        patch("rotate_halves", lambda x, pos, rot: x)
    elif mistake == "neighbours":
        def turn(x, pos, rot):
            n = rot["dims"] // 2
            y = x.copy()
            y[..., :n], y[..., n:2 * n] = x[..., 0:2 * n:2], x[..., 1:2 * n:2]
            return real["rotate_halves"](y, pos, rot)
        patch("rotate_halves", turn)
    elif mistake == "rotated_key_normed":
        def cache(h, w, p, mx, eps):
            c, k = real["latents"](h, w, p, mx, eps)
            return c, orc.unit_rms(k, eps)
        patch("latents", cache)
    elif mistake == "yarn_gain":
        patch("rotary_frequencies", lambda d, b, s=None: (real["rotary_frequencies"](d, b, s)[0], 1.0))
    elif mistake == "yarn_freq":
        patch("rotary_frequencies", lambda d, b, s=None: (real["rotary_frequencies"](d, b)[0], real["rotary_frequencies"](d, b, s)[1]))
    elif mistake == "kv_from":
        del cfg["layers"][3]["mixer"]["kv_from"]            # the layer's own input through the other layer's projections
        w |= {"l3." + n[3:]: t for n, t in w.items() if n.startswith("l0.mix.dkv")}
    elif mistake == "shared_own_rank":
        cfg["layers"][7]["mixer"]["kv_from"] = 5
        w["l7.mix.uk"] = np.tile(w["l5.mix.uk"], (3, 1))[:40]
    elif mistake == "floor":
        memory(floor=False)
    elif mistake in ("input_cap", "forget_cap"):
        calls = []
        patch("capped", lambda z, cap: (calls.append(0), z if (len(calls) % 2 == 1) == (mistake == "input_cap") else real["capped"](z, cap))[1])
    elif mistake == "forget_gate":
        memory(cap_f=lambda f: 0 * f)
    elif mistake == "key_scale":
        memory(key=0.2)
    elif mistake == "mlstm_norm":
        change("mix.norm", np.ones_like)
    elif mistake == "mlstm_gate":
        for i in (2, 4):
            change(f"l{i}.mix.g")
    elif mistake == "state_lost":
        patch("mlstm_recurrence", lambda *a: cut(real["mlstm_recurrence"], *a))
    elif mistake == "candidate":
        patch("mingru_recurrence", lambda z, u: (lambda c: (np.stack([sum((z[s] * c[s] * np.prod(1 - z[s + 1:t + 1], axis=0)) for s in range(t + 1)) for t in range(len(z))]), None))(u))
    elif mistake == "gru_state_lost":
        patch("mingru_recurrence", lambda z, u: cut(real["mingru_recurrence"], z, u))
    elif mistake == "gru_gate":
        for i in (1, 6):
            change(f"l{i}.mix.g", lambda t: t * 0.5)
    elif mistake == "gru_bias":
        change("mix.x.b")
    elif mistake == "conv":
        patch("causal_conv", lambda h, c: h)
    elif mistake == "conv_order":
        patch("causal_conv", lambda h, c: real["causal_conv"](h, c[:, ::-1]))
    elif mistake == "conv_lost":
        patch("causal_conv", lambda h, c: np.concatenate([real["causal_conv"](h[i:i + 40], c) for i in range(0, len(h), 40)]))
    elif mistake == "conv_alone":
        patch("causal_conv", lambda h, c: real["causal_conv"](h, c) - h)
    elif mistake == "streams_in":
        patch("streams_in", lambda x, w, p: x.sum(axis=0))
    elif mistake == "streams_transposed":
        patch("streams_out", lambda x, y, w, p: real["streams_out"](x, y, {p + "mix": w[p + "mix"].T, p + "out": w[p + "out"]}, p))
    elif mistake == "streams_out":
        change("hc1.out", np.ones_like)
    elif mistake == "bigram":
        change("bigram")
    elif mistake == "bigram_first":
        patch("bigram_rows", lambda ids, b, p, c: [0] + real["bigram_rows"](ids, b, p, c)[1:])
    elif mistake == "bigram_order":
        patch("bigram_rows", lambda ids, b, p, c: real["bigram_rows"](ids, b, c, p))
    elif mistake == "positions":
        w["pos"] = np.roll(w["pos"], 1, axis=0)
    elif mistake in ("xielu_up", "xielu_down"):
        at = 0 if mistake == "xielu_up" else 1
        change("mlp.act", lambda t: np.where(np.arange(2) == at, 0.0, t))
    elif mistake == "xielu_slope":
        patch("xielu", lambda z, p, q: real["xielu"](z, p, q) - np.where(z > 0, 0.0, 0.5 * (np.expm1(np.minimum(z, 0)) - z)))
    elif mistake == "zero_centred":
        change("norm1", lambda t: t - 1.0)
    moved = bu.err(orc.forward(cfg, w, ids), want)
    assert moved > 0.01, moved
