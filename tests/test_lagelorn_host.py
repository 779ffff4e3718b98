"""Lagelorn without a GPU: configuration, registry, distance buckets, and the oracle against itself."""
import json

import numpy as np
import pytest

import lagelorn_util as lu
from oracle import lagelorn_oracle as orc
from proxy_inference_engine_amd.models import utils as mu
from proxy_inference_engine_amd.models.lagelorn import ModelArgs
from proxy_inference_engine_amd.models.lagelorn.language import distance_buckets


def test_config_is_read_layer_by_layer():
    a = ModelArgs(**json.loads(json.dumps(lu.CONFIGS["mixed"])))
    assert [lay.type for lay in a.layers] == [m[0] for m, _ in lu.MIXED]
    assert a.layers[1].mlp is None and a.layers[2].mixer.conv == 5 and a.layers[2].mixer.kv_heads == 2 and a.layers[2].mlp.ff == 33
    assert a.layers[3].mixer.left.mask.size == 33 and a.layers[4].mixer.left.mask is None and (a.layers[3].mixer.left_scale, a.layers[3].mixer.right_scale) == (1.2, 0.5)
    assert a.layers[3].mixer.left.bias_max == 40 and a.layers[3].mixer.right.dim == 33
    assert (a.postln_alpha, a.logit_softcap, a.token_side.dim, a.max_positions) == (1.7, 4.0, 16, 640)


def test_registry_knows_the_design():
    assert "Lagelorn" in mu._ARCHITECTURES


@pytest.mark.parametrize("rows", [2, 3, 4, 12, 16, 31, 32, 64])
def test_distance_buckets(rows):
    """The table by distance: every entry, and everything behind its end."""
    for far in (rows // 2 + 1, rows, 40, 100.5, 128, 1000):
        if far <= rows // 2:
            continue
        got = distance_buckets(rows, far)
        assert got == [orc.distance_bucket(n, rows, far) for n in range(len(got))] and got == sorted(got)
        assert all(orc.distance_bucket(n, rows, far) == got[-1] == rows - 1 for n in range(len(got), len(got) + 300)) and got[-2] < rows - 1
    with pytest.raises(ValueError):
        distance_buckets(rows, rows // 2)


# ------------------------------------------------------------------ the oracle against itself
def test_oracle_recurrences_continue_from_their_states():
    rng = np.random.default_rng(0)
    q, k, v = rng.normal(size=(11, 2, 5)), rng.normal(size=(11, 2, 5)), rng.normal(size=(11, 2, 3))
    g, b = rng.random((11, 2)), rng.random((11, 2))
    whole, end = orc.gated_delta_recurrence(q, k, v, g, b)
    first, state = orc.gated_delta_recurrence(q[:4], k[:4], v[:4], g[:4], b[:4])
    rest, end2 = orc.gated_delta_recurrence(q[4:], k[4:], v[4:], g[4:], b[4:], state)
    assert np.allclose(np.concatenate([first, rest]), whole) and np.allclose(end, end2)
    r, k, v, w, u = (rng.normal(size=(11, 2, 4)) for _ in range(5))
    w, u = rng.random((11, 2, 4)), u[0]
    whole, end = orc.rwkv_recurrence(r, k, v, w, u)
    first, state = orc.rwkv_recurrence(r[:4], k[:4], v[:4], w[:4], u)
    rest, end2 = orc.rwkv_recurrence(r[4:], k[4:], v[4:], w[4:], u, state)
    assert np.allclose(np.concatenate([first, rest]), whole) and np.allclose(end, end2)


def test_oracle_delta_rule_replaces_what_a_key_holds():
    """A step of one: the state answers a unit key with the value written last, whatever stood there, and what was written under an orthogonal key has only decayed."""
    e = np.eye(4)
    k, v = np.stack([e[0], e[1], e[0]])[:, None], np.array([[1.0, 2.0], [3.0, 4.0], [5.0, 6.0]])[:, None]
    o, S = orc.gated_delta_recurrence(k, k, v, np.array([[1.0], [0.5], [0.5]]), np.ones((3, 1)))
    assert np.allclose(o[:, 0], v[:, 0]) and np.allclose(S[0], [[5, 6], [1.5, 2], [0, 0], [0, 0]])


def test_oracle_time_mixing_is_a_sum_over_the_past():
    rng = np.random.default_rng(1)
    r, k, v, w, u = rng.normal(size=(7, 1, 4)), rng.normal(size=(7, 1, 4)), rng.normal(size=(7, 1, 4)), rng.random((7, 1, 4)), rng.normal(size=(1, 4))
    o, _ = orc.rwkv_recurrence(r, k, v, w, u)
    t = 6
    want = (r[t, 0] * u[0] * k[t, 0]).sum() * v[t, 0] + sum((r[t, 0] * np.prod(w[s + 1:t, 0], axis=0) * k[s, 0]).sum() * v[s, 0] for s in range(t))
    assert np.allclose(o[t, 0], want)


def test_oracle_convolution_is_causal():
    x, w = np.zeros((6, 2)), np.array([[1.0, 2.0, 3.0], [0.0, 0.0, 0.5]])
    x[2] = 1.0
    assert orc.causal_conv(x, w).tolist() == [[0, 0], [0, 0], [3, 0.5], [2, 0], [1, 0], [0, 0]]


def test_oracle_chunks_count_from_the_start():
    assert orc.visible(5, 2).astype(int).tolist() == [[1, 0, 0, 0, 0], [1, 1, 0, 0, 0], [0, 0, 1, 0, 0], [0, 0, 1, 1, 0], [0, 0, 0, 0, 1]]


def test_oracle_token_shift():
    assert orc.token_shift(np.array([[1.0], [3.0], [7.0]]), np.array([0.25])).tolist() == [[0.75], [2.5], [6.0]]


MISTAKES = ["alpha", "norm_before", "positions", "side", "side_gate", "side_norm", "side_layer", "softcap", "conv", "conv_order", "conv_silu", "conv_lost", "unit_q", "q_scale", "unit_k", "beta", "decay",
            "softplus", "write_before_read", "delta_state_lost", "delta_groups", "delta_norm", "delta_gate", "delta_gate_sigmoid", "left_scale", "right_scale", "q_bias", "k_bias", "value_bias", "value_norm", "norm_per_head",
            "score_scale", "bias_scaled", "bias_shifted", "bias_heads", "bias_far", "chunk", "chunk_shifted", "window", "sink", "sink_scaled", "left_groups", "shift", "shift_lost", "mu", "rwkv_decay", "w0", "w1_tanh", "bonus", "bonus_kept",
            "read_after", "rwkv_state_lost", "rwkv_norm", "rwkv_gate", "rwkv_head_norm", "ff_bias", "ff_up_bias", "ff_down_bias", "ff_gelu"]


@pytest.mark.parametrize("mistake", MISTAKES)
def test_oracle_mistakes_show(mistake, monkeypatch):
    """With weights like those of the device tests, every mechanism left out or replaced moves the logits: by several hundred times what the 32-bit tests allow."""
    cfg = json.loads(json.dumps(lu.CONFIGS["mixed"]))
    if mistake == "q_scale":   # (the head's norm takes any factor out again, unless its epsilon counts)
        cfg["norm"]["eps"] = 0.3
    w, ids = lu.as_numpy(lu.weights(cfg, seed=3, q_gain=1.5)), lu.tokens(cfg, 120)
    want = orc.forward(cfg, w, ids)
    names = ("unit_vectors", "gated_delta_recurrence", "causal_conv", "silu", "softplus", "gelu", "norm_of_sum", "side_input", "softcap", "distance_bucket", "visible", "sink_softmax", "project_keys",
             "token_shift", "rwkv_recurrence", "rwkv_decay", "unit_rms", "delta_decay", "attention", "embed")
    real = {n: getattr(orc, n) for n in names}
    patch = lambda name, f: monkeypatch.setattr(orc, name, f)  # noqa: E731

    def change(end, f=np.zeros_like):
        found = [n for n in w if n.endswith(end)]
        assert found
        for n in found:
            w[n] = f(w[n])

    def cut(f, args, n, *rest):
        return np.concatenate([f(*(a[i:i + 40] for a in args), *rest)[0] for i in range(0, n, 40)]), None

    def delta_with(q=lambda q: q, k=lambda k: k, g=lambda g: g, b=lambda b: b):
        patch("gated_delta_recurrence", lambda *a: real["gated_delta_recurrence"](q(a[0]), k(a[1]), a[2], g(a[3]), b(a[4])))

    if mistake == "alpha":
        patch("norm_of_sum", lambda x, y, n, alpha, eps: real["norm_of_sum"](x, y, n, 1.0, eps))
    elif mistake == "norm_before":
        patch("norm_of_sum", lambda x, y, n, alpha, eps: alpha * x + orc.rms_norm(y, n, eps))
    elif mistake == "positions":
        w["pos"] = np.roll(w["pos"], 1, axis=0)
    elif mistake == "side":
        patch("side_input", lambda x, *a: x)
    elif mistake == "side_gate":
        change("side.gate")
    elif mistake == "side_norm":
        change("side.norm", np.ones_like)
    elif mistake == "side_layer":
        w["side.embed"] = np.roll(w["side.embed"], 16, axis=1)
    elif mistake == "softcap":
        patch("softcap", lambda z, cap: z)
    elif mistake == "conv":
        patch("causal_conv", lambda x, c: x)
    elif mistake == "conv_order":
        patch("causal_conv", lambda x, c: real["causal_conv"](x, c[:, ::-1]))
    elif mistake == "conv_silu":
        calls = []
        patch("silu", lambda z: (calls.append(0), z if z.shape[1] in (60, 84, 32, 160) and len(calls) % 4 else real["silu"](z))[1])
    elif mistake == "conv_lost":
        patch("causal_conv", lambda x, c: np.concatenate([real["causal_conv"](x[i:i + 40], c) for i in range(0, len(x), 40)]))
    elif mistake in ("unit_q", "unit_k"):
        calls = []
        patch("unit_vectors", lambda x: (calls.append(0), x if (len(calls) % 2 == 1) == (mistake == "unit_q") else real["unit_vectors"](x))[1])
    elif mistake == "q_scale":
        delta_with(q=lambda q: 4.0 * q)
    elif mistake == "beta":
        delta_with(b=np.ones_like)
    elif mistake == "decay":
        delta_with(g=np.ones_like)
    elif mistake == "softplus":
        patch("softplus", np.exp)
    elif mistake == "write_before_read":   # the read-out misses the current token's write
        def run(q, k, v, g, b, state=None):
            S, o = np.zeros((q.shape[1], q.shape[2], v.shape[2])), np.empty_like(v)
            for t in range(len(q)):
                S = g[t][:, None, None] * S
                o[t] = np.einsum("hde,hd->he", S, q[t])
                S = S + k[t][:, :, None] * (b[t][:, None] * (v[t] - np.einsum("hde,hd->he", S, k[t])))[:, None, :]
            return o, None
        patch("gated_delta_recurrence", run)
    elif mistake == "delta_state_lost":
        patch("gated_delta_recurrence", lambda *a: cut(real["gated_delta_recurrence"], a, len(a[0])))
    elif mistake == "delta_groups":
        delta_with(q=lambda q: q[:, [0, 2, 1, 3]] if q.shape[1] == 4 else q)
    elif mistake == "delta_norm":
        change("mix.norm", np.ones_like)
    elif mistake == "delta_gate":
        for i in (1, 2):
            change(f"l{i}.mix.g", lambda t: 0.5 * t)
    elif mistake == "delta_gate_sigmoid":
        patch("silu", lambda z: orc.sigmoid(z) if z.shape[1] in (84, 160) else real["silu"](z))
    elif mistake in ("left_scale", "right_scale"):
        for i in (0, 3, 4):
            cfg["layers"][i]["mixer"][mistake] = 1.0
    elif mistake == "q_bias":
        change("left.q.b")
    elif mistake == "k_bias":
        change("left.k.b")
    elif mistake in ("value_bias", "value_norm"):
        def keys(h, w, p, mx, eps):
            k, v = real["project_keys"](h, w, p, mx, eps)
            return k, k if mistake == "value_norm" else v - w[p + "k.b"].reshape(v.shape[1:])
        patch("project_keys", keys)
    elif mistake == "norm_per_head":
        def keys(h, w, p, mx, eps):
            k, v = real["project_keys"](h, w, p, mx, eps)
            return orc.unit_rms(v, eps) * w[p + "k.norm"].reshape(v.shape[1:]), v
        patch("project_keys", keys)
    elif mistake == "score_scale":
        cfg["layers"][3]["mixer"]["left"]["scale"] = 9 ** -0.5
    elif mistake == "bias_scaled":
        change("left.rel", lambda t: 0.3 * t)
    elif mistake == "bias_shifted":
        patch("distance_bucket", lambda n, rows, far: real["distance_bucket"](n + 1, rows, far))
    elif mistake == "bias_heads":
        change("left.rel", lambda t: t[:, ::-1])
    elif mistake == "bias_far":
        patch("distance_bucket", lambda n, rows, far: real["distance_bucket"](n, rows, 2 * far))
    elif mistake == "chunk":
        patch("visible", lambda n, c: real["visible"](n, None))
    elif mistake == "chunk_shifted":
        patch("visible", lambda n, c: real["visible"](n + 1, c)[1:, 1:])
    elif mistake == "window":
        patch("visible", lambda n, c: real["visible"](n, None) & (np.arange(n)[:, None] - np.arange(n)[None, :] < (c or n)))
    elif mistake == "sink":
        patch("sink_softmax", lambda s, m, sink: real["sink_softmax"](s, m, -1e30))
    elif mistake == "sink_scaled":
        patch("sink_softmax", lambda s, m, sink: real["sink_softmax"](s, m, 0.2 * sink))
    elif mistake == "left_groups":
        patch("project_keys", lambda *a: tuple(t[:, ::-1] for t in real["project_keys"](*a)))
    elif mistake == "shift":
        patch("token_shift", lambda h, m: h)
    elif mistake == "shift_lost":
        patch("token_shift", lambda h, m: np.concatenate([real["token_shift"](h[i:i + 40], m) for i in range(0, len(h), 40)]))
    elif mistake == "mu":
        change("mu.k", lambda t: 1.0 - t)
    elif mistake == "rwkv_decay":
        patch("rwkv_decay", lambda x, w, p: np.ones((len(x), len(w[p + "w0"]))))
    elif mistake == "w0":
        change("right.w0", lambda t: t + 1.0)
    elif mistake == "w1_tanh":
        patch("rwkv_decay", lambda x, w, p: np.exp(-np.exp((x @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"])))
    elif mistake == "bonus":
        change("right.u", np.ones_like)
    elif mistake == "bonus_kept":
        patch("rwkv_recurrence", lambda r, k, v, d, u: real["rwkv_recurrence"](r, k * u, v, d, np.ones_like(u)))
    elif mistake == "read_after":   # the decay is taken before the read-out
        patch("rwkv_recurrence", lambda r, k, v, d, u: (lambda o, own: (o + own, None))(real["rwkv_recurrence"](r * d, k, v, d, np.zeros_like(u))[0], ((r * u * k).sum(-1, keepdims=True) * v)))
    elif mistake == "rwkv_state_lost":
        patch("rwkv_recurrence", lambda *a: cut(real["rwkv_recurrence"], a[:4], len(a[0]), a[4]))
    elif mistake == "rwkv_norm":
        change("right.norm", np.ones_like)
    elif mistake == "rwkv_gate":
        change("right.g", lambda t: 0.5 * t)
    elif mistake == "rwkv_head_norm":
        patch("unit_rms", lambda x, eps: x if x.ndim == 3 and x.shape[1] in (2, 5) else real["unit_rms"](x, eps))
    elif mistake == "ff_bias":
        change("gate.b")
    elif mistake == "ff_up_bias":
        change("up.b")
    elif mistake == "ff_down_bias":
        change("down.b")
    elif mistake == "ff_gelu":
        patch("gelu", lambda z: z * orc.sigmoid(1.702 * z))
    moved = lu.err(orc.forward(cfg, w, ids), want)
    assert moved > 0.01, moved
