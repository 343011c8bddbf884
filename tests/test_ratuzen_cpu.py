"""CPU-side checks of the Ratuzen design: the checkpoint folder the writer in synth.py makes, what the host's loader refuses before it
touches a device, and the plain oracle's own consistency (prompt pass against portions and token-by-token feeding, chunk edges, the two
rotations and their frequency scalings, the recurrences, the normed pair). Nothing here needs a GPU; everything that computes on the
product path is in test_ratuzen_gpu.py."""
import json
import math

import numpy as np
import pytest


@pytest.fixture(scope="module")
def synth(pkg):
    from tinyllama_cpp_amd import synth as s
    return s


def tiny_config(synth):
    K, C, D, L = synth.ratuzen_chunked, synth.ratuzen_causal, synth.ratuzen_delta, synth.ratuzen_layer
    return synth.ratuzen_config(24, 31, [
        L("parallel", K(4, 2, 6, 5, 7, 2, 8, 6, [0.9, 0.5], rot_dims=4, scaling=(4.0, 1.0, 4.0, 32)), 10),
        L("delta", D(4, 2, 8, 6, conv=3)),
        L("parallel_2", C(4, 2, 8, 6, 3, 6, 5, tau=4.0, rot_dims=6, factor=2.0), 7)])


def test_checkpoint_names(synth, tmp_path):
    cfg = tiny_config(synth)
    tensors = synth.build_ratuzen(cfg, 3, rank=5)
    synth.write_stack_dir(str(tmp_path), cfg, tensors)
    assert json.load(open(tmp_path / "config.json")) == cfg
    assert {"embed", "head", "final.norm", "l0.norm1", "l0.norm2", "l0.mix.left.q", "l0.mix.left.v.b", "l0.mix.left.o", "l0.mix.left.out",
            "l0.mix.right.q", "l0.mix.right.g", "l0.mix.right.norm", "l0.mix.right.out", "l0.mlp.gate", "l1.mix.q.conv", "l1.mix.A_log",
            "l1.mix.dt_bias", "l1.mix.g", "l2.mix.left.q.norm", "l2.mix.left.g", "l2.mix.right.a1", "l2.mix.right.a2", "l2.mix.right.a2.b"} <= set(tensors)
    assert "l1.norm2" not in tensors and "l2.mix.left.q.b" not in tensors and "l0.mix.left.q.norm" not in tensors
    assert tensors["l0.mix.right.norm"].shape == (2 * 6,) and tensors["l2.mix.right.norm"].shape == (5,)
    assert tensors["l2.mix.left.g"].shape == (4, 24) and tensors["l2.mix.right.a2"].shape == (18, 5)
    assert tensors["l1.mix.q"].shape == (2 * 8, 24) and tensors["l1.mix.v.conv"].shape == (4 * 6, 3)


def test_oracle_prompt_equals_portions_and_tokens(synth):
    from oracle.ratuzen_oracle import RatuzenOracle
    cfg = tiny_config(synth)
    orc = RatuzenOracle(cfg, synth.build_ratuzen(cfg, 5))
    toks = list(np.random.default_rng(0).integers(0, 31, 24))
    whole = orc.forward(toks)
    orc.reset()
    parts = np.concatenate([orc.forward(toks[:6]), orc.forward(toks[6:8])] + [orc.forward([t]) for t in toks[8:]])
    assert np.allclose(whole, parts, rtol=1e-9, atol=1e-11)
    orc.reset()
    assert np.allclose(orc.forward(toks), whole, rtol=0, atol=0)               # nothing survives a reset
    cfg2 = dict(cfg, logit_scale=2 * cfg["logit_scale"])
    assert np.allclose(RatuzenOracle(cfg2, synth.build_ratuzen(cfg, 5)).forward(toks), 2 * whole)


def test_oracle_chunks():
    from oracle.ratuzen_oracle import first_visible, softmax_attention
    rng = np.random.default_rng(1)
    n, dim = 12, 4
    q, k, v = rng.standard_normal((n, 2, dim)), rng.standard_normal((n, 1, dim)), rng.standard_normal((n, 1, 3))
    pos = np.arange(n)
    plain = softmax_attention(q, k, v, 0.5, pos)
    assert np.allclose(softmax_attention(q, k, v, 0.5, pos, chunk=n), plain)             # one chunk: nothing changes
    assert np.allclose(softmax_attention(q, k, v, 0.5, pos, chunk=1)[:, 0], v[:, 0])     # chunks of one see themselves only
    out = softmax_attention(q, k, v, 0.5, pos, chunk=5)
    assert np.allclose(out[:5], plain[:5]) and np.allclose(out[5, 0], v[5, 0]) and np.allclose(out[10, 0], v[10, 0])
    fresh = softmax_attention(q[5:10], k[5:10], v[5:10], 0.5, np.arange(5))              # a chunk is a sequence of its own (without rotation)
    assert np.allclose(out[5:10], fresh)
    assert [first_visible(i, 5) for i in (0, 4, 5, 9, 10)] == [0, 0, 5, 5, 10] and first_visible(9, 0) == 0


def test_oracle_rotations():
    from oracle.ratuzen_oracle import frequencies, rotate
    rng = np.random.default_rng(2)
    x = rng.standard_normal((6, 2, 8))
    pos = np.arange(100, 106)
    f = frequencies({"base": 100.0, "dims": 6})
    assert np.allclose(f, [1.0, 100.0 ** (-1 / 3), 100.0 ** (-2 / 3)])
    for halves in (False, True):
        y = rotate(x, pos, f, halves)
        assert np.allclose((y * y).sum(-1), (x * x).sum(-1)) and np.allclose(y[..., 6:], x[..., 6:])
        # only the distance of two positions counts in their product
        a = (rotate(x, pos, f, halves) * rotate(x[::-1], pos - 3, f, halves)).sum(-1)
        b = (rotate(x, pos + 50, f, halves) * rotate(x[::-1], pos + 47, f, halves)).sum(-1)
        assert np.allclose(a, b)
    # the two layouts are the same rotation under a permutation of the dimensions
    perm = [0, 2, 4, 1, 3, 5, 6, 7]
    assert np.allclose(rotate(x[..., perm], pos, f, True), rotate(x, pos, f, False)[..., perm])
    assert np.allclose(frequencies({"base": 100.0, "dims": 6, "scaling": {"factor": 4.0}}), f / 4.0)
    sc = {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 40}
    g = frequencies({"base": 1000.0, "dims": 8, "scaling": sc})
    f = frequencies({"base": 1000.0, "dims": 8})
    for a, b in zip(g, f):
        length = 2 * math.pi / b
        if length < 10:
            assert a == b
        elif length > 40:
            assert np.isclose(a, b / 8)
        else:
            assert b / 8 < a < b
    edge = 2 * math.pi / 10.0                                                  # the blend joins both ranges without a step
    s = lambda length: (40 / length - 1) / 3
    assert np.isclose((1 - s(10.0)) * edge / 8 + s(10.0) * edge, edge) and np.isclose(s(40.0), 0.0)


def test_oracle_recurrences(synth):
    from oracle.ratuzen_oracle import RatuzenOracle, gated_delta_rule, linear_recurrence
    rng = np.random.default_rng(3)
    d, vd, n = 4, 3, 6
    q, k, v = rng.standard_normal((n, d)), rng.standard_normal((n, d)), rng.standard_normal((n, vd))
    S = np.zeros((d, vd))
    o = linear_recurrence(q, k, v, 0.0, S)                                       # nothing is kept: o = v (k . q)
    assert np.allclose(o, v * (k * q).sum(-1, keepdims=True))
    S = np.zeros((d, vd))
    o = linear_recurrence(q, k, v, 1.0, S)                                       # everything is kept: plain linear attention
    w = np.tril(q @ k.T)
    assert np.allclose(o, w @ v)
    S = np.zeros((d, vd))
    o = linear_recurrence(q, k, v, 0.5, S)
    decay = 0.5 ** (np.arange(n)[:, None] - np.arange(n)[None, :])
    assert np.allclose(o, (w * decay) @ v)
    S, S2 = np.zeros((d, vd)), np.zeros((d, vd))                                 # a decay per channel acts on the rows of its key channel
    rate = np.array([0.0, 1.0, 0.5, 0.9])
    linear_recurrence(q, k, v, rate, S)
    linear_recurrence(q[:, 1:2], k[:, 1:2], v, 1.0, S2[1:2])
    assert np.allclose(S[1], S2[1]) and np.allclose(S[0], k[-1, 0] * v[-1])
    S = np.zeros((d, vd))
    e = np.zeros((1, d))
    e[0, 2] = 1.0
    assert np.allclose(gated_delta_rule(e, e, v[:1], np.ones(1), np.ones(1), S)[0], v[0])
    assert np.allclose(gated_delta_rule(e, e, v[1:2], np.ones(1), np.array([0.5]), S)[0], v[1])   # decay first, then the old content is replaced
    # the norms of a pair make it blind to the size of either output
    cfg = tiny_config(synth)
    cfg["norm"]["eps"] = 1e-12
    t = synth.build_ratuzen(cfg, 1)
    a = RatuzenOracle(cfg, t).forward([1, 2, 3, 4])
    t["l0.mix.left.o"] = synth.to_bf16(synth.from_bf16(t["l0.mix.left.o"]) * 4.0)
    assert np.allclose(RatuzenOracle(cfg, t).forward([1, 2, 3, 4]), a)


@pytest.fixture(scope="module")
def hostapi(pkg):
    from tinyllama_cpp_amd import hostapi as h
    h.lib()
    return h


def test_loader_refusals(synth, hostapi, tmp_path):
    cfg = tiny_config(synth)
    tensors = synth.build_ratuzen(cfg, 7)

    def refused(name, change, match):
        bad = json.loads(json.dumps(cfg))
        change(bad)
        synth.write_stack_dir(str(tmp_path / name), bad, tensors)
        with pytest.raises(hostapi.TlHostError, match=match):
            hostapi.Session(str(tmp_path / name), 0, 64)

    refused("type", lambda c: c["layers"][1].update(type="delta_2"), "layers\\[1\\].*delta_2")
    refused("ff", lambda c: c["layers"][0]["mlp"].update(kind="moe"), "layers\\[0\\].*moe")
    refused("decays", lambda c: c["layers"][0]["mixer"]["right"].update(decay=[0.5]), "layers\\[0\\].*1 decays for 2 heads")
    refused("scale", lambda c: c.pop("logit_scale"), "logit_scale")
    refused("tau", lambda c: c["layers"][2]["mixer"]["right"].pop("tau"), "tau")
    del tensors["l2.mix.right.a1"]
    refused("a1", lambda c: None, "l2.mix.right.a1")
