"""CPU-side checks of the Madudra design: the checkpoint folder the writer in synth.py makes, what the host's loader refuses
before it touches a device, and the plain oracle's own consistency. Nothing here needs a GPU; everything that computes on the
product path is in test_madudra_gpu.py."""
import json
import math

import numpy as np
import pytest


@pytest.fixture(scope="module")
def synth(pkg):
    from tinyllama_cpp_amd import synth as s
    return s


@pytest.fixture(scope="module")
def hostapi(pkg):
    from tinyllama_cpp_amd import hostapi as h
    h.lib()
    return h


def tiny_config(synth, streams=2):
    A, M, E, L = synth.madudra_latent, synth.madudra_mamba, synth.madudra_moe, synth.madudra_layer
    return synth.madudra_config(24, 31, [
        L("mamba2", M(4, 6, 5, groups=2, conv=3, norm_groups=4), E(4, 2, 7, scale=1.5)),
        L("latent_attention", A(3, 6, 4, 5, 11, 9, 7, scaling=(2.0, 16, 4.0, 1.0)), None),
        L("latent_attention", A(2, 8, 4, 6, 10, 9, 4, scaling=(2.0, 16, 4.0, 1.0), kv_from=1), E(3, 1, 10))], streams=streams)


def test_checkpoint_names(synth, tmp_path):
    cfg = tiny_config(synth)
    t = synth.build_madudra(cfg, 3)
    synth.write_stack_dir(str(tmp_path), cfg, t)
    assert json.load(open(tmp_path / "config.json")) == cfg
    assert {"embed", "head", "final.norm", "l0.norm1", "l0.hc1.in", "l0.hc2.mix", "l0.mix.in", "l0.mix.conv", "l0.mix.conv.b", "l0.mix.dt_bias",
            "l0.mix.A_log", "l0.mix.D", "l0.mix.norm", "l0.mix.o", "l0.mlp.router", "l0.mlp.e3.up", "l0.mlp.e3.down", "l1.mix.dkv",
            "l1.mix.dkv.norm", "l1.mix.g", "l2.mix.uq", "l2.mix.uk", "l2.mix.uv"} <= set(t)
    assert "l0.mlp.e0.gate" not in t and "l2.mix.dkv" not in t and "l1.norm2" not in t and "l1.hc2.in" not in t
    assert not any(k.endswith("norm1.b") or k.endswith("norm2.b") for k in t)
    assert t["l0.mix.in"].shape == (2 * 24 + 2 * 2 * 5 + 4, 24) and t["l0.mix.conv"].shape == (24 + 2 * 2 * 5, 3)
    assert t["l1.mix.g"].shape == (15, 24) and t["l0.hc1.mix"].shape == (2, 2)


def test_oracle_prompt_equals_portions_and_tokens(synth):
    from oracle.madudra_oracle import MadudraOracle
    cfg = tiny_config(synth)
    orc = MadudraOracle(cfg, synth.build_madudra(cfg, 5))
    toks = list(np.random.default_rng(0).integers(0, 31, 24))
    whole = orc.forward(toks)
    orc.reset()
    parts = np.concatenate([orc.forward(toks[:6]), orc.forward(toks[6:8])] + [orc.forward([t]) for t in toks[8:]])
    assert np.allclose(whole, parts, rtol=1e-9, atol=1e-11)
    orc.reset()
    assert np.allclose(orc.forward(toks), whole, rtol=0, atol=0)


def test_oracle_streams():
    from oracle.madudra_oracle import streams_in, streams_out
    rng = np.random.default_rng(1)
    xs, y = rng.standard_normal((4, 3, 5)), rng.standard_normal((4, 5))
    # the identity with unit weights is the plain residual in every stream
    assert np.allclose(streams_out(xs, y, np.eye(3), np.ones(3), 0.5), xs + 0.5 * y[:, None])
    # one entry of the mix moves one stream into one other: [from, to]
    mix = np.zeros((3, 3))
    mix[2, 0] = 2.0
    out = streams_out(xs, y, mix, np.array([0.0, 1.0, 0.0]), 1.0)
    assert np.allclose(out[:, 0], 2.0 * xs[:, 2]) and np.allclose(out[:, 1], y) and np.allclose(out[:, 2], 0.0)
    assert np.allclose(streams_in(xs, np.array([0.0, -1.0, 0.0])), -xs[:, 1])


def test_oracle_rotation():
    from oracle.madudra_oracle import rotary_frequencies, rotate_halves
    f, ms = rotary_frequencies(8, 100.0)
    assert ms == 1.0 and np.allclose(f, 100.0 ** (-np.arange(4) / 4.0))
    g, ms = rotary_frequencies(8, 100.0, {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0})
    assert math.isclose(ms, 0.1 * math.log(4.0) + 1.0)
    assert math.isclose(g[0], f[0]) and math.isclose(g[-1], f[-1] / 4.0)     # fast turns stay, slow ones stretch
    x = np.random.default_rng(2).standard_normal((6, 2, 11))
    r = rotate_halves(x, np.arange(6), 8, f, 1.0)
    assert np.allclose(r[0], x[0]) and np.allclose(r[..., 8:], x[..., 8:])
    assert np.allclose(r[..., :4] ** 2 + r[..., 4:8] ** 2, x[..., :4] ** 2 + x[..., 4:8] ** 2)  # the pairs are (i, i + 4)
    # only the distance counts in a product of two rotated vectors
    a, b = x[0, 0, :8], x[1, 0, :8]
    turn = lambda v, p: rotate_halves(v[None], [p], 8, f, 1.0)[0]
    assert math.isclose(turn(a, 9) @ turn(b, 4), turn(a, 105) @ turn(b, 100), rel_tol=1e-9)


def test_oracle_window_and_router():
    from oracle.madudra_oracle import route_softmax, softmax_attention
    rng = np.random.default_rng(3)
    q, k, v = rng.standard_normal((12, 2, 4)), rng.standard_normal((12, 2, 4)), rng.standard_normal((12, 2, 3))
    pos = np.arange(12)
    plain = softmax_attention(q, k, v, 0.5, pos)
    assert np.allclose(softmax_attention(q, k, v, 0.5, pos, window=12), plain)
    assert np.allclose(softmax_attention(q, k, v, 0.5, pos, window=1), v)
    k2 = k.copy()
    k2[:5] = 99.0
    assert np.allclose(softmax_attention(q, k2, v, 0.5, pos, 3)[7:], softmax_attention(q, k, v, 0.5, pos, 3)[7:])
    z = np.array([1.0, 3.0, -2.0, 2.0])
    ids, w = route_softmax(z, 2, 2.0)
    assert list(ids) == [1, 3] and np.allclose(w, 2.0 * np.exp(z[[1, 3]]) / np.exp(z).sum())


def test_oracle_state_space():
    from oracle.madudra_oracle import gated_part_norm, state_space
    rng = np.random.default_rng(4)
    n, N, vd = 6, 4, 3
    x, B, C, dt = rng.standard_normal((n, vd)), rng.standard_normal((n, N)), rng.standard_normal((n, N)), rng.uniform(0.1, 2.0, n)
    S = np.zeros((N, vd))
    y = state_space(x, B, C, dt, 0.7, 0.3, S)
    # the recurrence unrolled: y_i = sum_j exp(-rate (dt_(j+1) + .. + dt_i)) dt_j (C_i . B_j) x_j + D x_i
    for i in range(n):
        want = 0.3 * x[i] + sum(math.exp(-0.7 * dt[j + 1:i + 1].sum()) * dt[j] * (C[i] @ B[j]) * x[j] for j in range(i + 1))
        assert np.allclose(y[i], want)
    g = gated_part_norm(rng.standard_normal((2, 8)), np.full((2, 8), 50.0), 4, 0.0, np.ones(8))
    assert np.allclose((g.reshape(2, 4, 2) ** 2).mean(-1), 1.0)               # every part has a root mean square of its own


def test_loader_refusals(synth, hostapi, tmp_path):
    cfg = tiny_config(synth)
    tensors = synth.build_madudra(cfg, 7)

    def refused(name, change, match):
        bad = json.loads(json.dumps(cfg))
        change(bad)
        synth.write_stack_dir(str(tmp_path / name), bad, tensors)
        with pytest.raises(hostapi.TlHostError, match=match):
            hostapi.Session(str(tmp_path / name), 0, 64)

    refused("layer", lambda c: c["layers"][1].update(type="convolution"), "layers\\[1\\].*convolution")
    refused("ff", lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "layers\\[0\\].*sparse")
    refused("cache", lambda c: c["layers"][2]["mixer"].update(kv_from=2), "kv_from")
    refused("streams", lambda c: c.pop("streams"), "streams")
    refused("none", lambda c: c.update(streams=0), "streams")
    refused("scale", lambda c: c["layers"][0]["mlp"]["router"].pop("scale"), "scale")
