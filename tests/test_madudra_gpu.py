"""Madudra layer-list models on the GPU against the plain float64 implementation in oracle/madudra_oracle.py.

Every test builds its own small configuration and random weights (synth.build_madudra). The product path is libtlhip.so
(operators, engine, decode graph) and, for generation, the C++ host (Session over a checkpoint folder). Exact mode
(three-term chunk GEMMs, FP32 GEMVs) is compared at FP32 tolerances, the bf16-activation mode at bf16 tolerances."""
import json
import math
import os

import numpy as np
import pytest

pytestmark = pytest.mark.gpu

FP32_TOL = 5e-5   # relative RMS per row, exact mode (observed ~1e-6)
BF16_TOL = 8e-2   # the same with bf16-rounded activations in the chunk GEMMs


def rel_rms(got, want):
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    d = got - want
    return float(np.sqrt((d * d).mean(-1)).max() / max(1e-12, np.sqrt((want * want).mean())))


def most_rows(got, want, q=0.5):
    """The error that a fraction q of the rows stays under: with bf16-rounded activations a token whose router decision is a
    close call takes another expert than the float64 model; such rows are off by design, most are not."""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    d = got - want
    return float(np.quantile(np.sqrt((d * d).mean(-1)), q) / max(1e-12, np.sqrt((want * want).mean())))


@pytest.fixture(scope="module")
def env(pkg):
    from tinyllama_cpp_amd import capi, engine, synth
    from oracle import madudra_oracle
    engine.init(0)
    return {"capi": capi, "engine": engine, "synth": synth, "oracle": madudra_oracle}


def small_config(synth, variant="mixed"):
    A, M, E, L = synth.madudra_latent, synth.madudra_mamba, synth.madudra_moe, synth.madudra_layer
    if variant == "mixed":  # unequal layers, shared latent caches under other windows, a layer without feed-forward
        return synth.madudra_config(72, 101, [
            L("latent_attention", A(6, 16, 8, 12, 40, 24, 11, base=5000.0, scaling=(4.0, 64, 8.0, 1.0)), E(8, 3, 24, scale=1.5)),
            L("mamba2", M(6, 12, 20, groups=3, conv=4, norm_groups=2), E(5, 1, 40, scale=2.5)),
            L("latent_attention", A(3, 8, 8, 20, 24, 24, 50, base=5000.0, scaling=(4.0, 64, 8.0, 1.0), kv_from=0), None),
            L("mamba2", M(2, 24, 8, groups=1, conv=3, norm_groups=6), None),
            L("latent_attention", A(4, 24, 12, 8, 16, 32, 37), E(4, 2, 16)),
            L("latent_attention", A(2, 16, 8, 16, 40, 24, 5, base=5000.0, scaling=(4.0, 64, 8.0, 1.0), kv_from=0), E(6, 6, 8, scale=0.5))],
            streams=3, residual_mult=0.6)
    if variant == "odd":  # nothing divisible by 4: every scalar fallback path; more streams than the unrolled kernels
        return synth.madudra_config(37, 53, [
            L("mamba2", M(3, 7, 5, groups=1, conv=2, norm_groups=7), E(5, 2, 11, scale=0.7)),
            L("latent_attention", A(3, 7, 6, 5, 13, 9, 9, scaling=(2.0, 32, 4.0, 1.0)), E(9, 4, 7, scale=3.0)),
            L("mamba2", M(5, 3, 9, groups=5, conv=5, norm_groups=1), E(3, 1, 5))], streams=5, residual_mult=1.3, eps=1e-3,
            embed_scale=0.5)
    if variant == "equal":  # values a model may happen to make equal or 1
        return synth.madudra_config(32, 64, [
            L("latent_attention", A(1, 32, 32, 32, 32, 32, 1, scale=1.0), E(1, 1, 32)),
            L("mamba2", M(1, 32, 32, groups=1, conv=1, norm_groups=1), E(2, 2, 32)),
            L("latent_attention", A(1, 32, 2, 32, 32, 32, 0, scale=0.2), None),
            L("mamba2", M(2, 1, 1, groups=2, conv=2, norm_groups=2), E(4, 4, 16))], streams=1, residual_mult=1.0, embed_scale=1.0)
    if variant == "wide":  # several tiles in every product, state sizes past one tile per wave, key sizes past the register path
        return synth.madudra_config(320, 300, [
            L("mamba2", M(8, 64, 130, groups=2, conv=4, norm_groups=4), E(16, 4, 96, scale=2.0)),
            L("latent_attention", A(8, 96, 40, 72, 96, 128, 130, base=250000.0, scaling=(4.0, 128, 16.0, 1.0)), E(8, 2, 64)),
            L("mamba2", M(4, 40, 300, groups=1, conv=4, norm_groups=2), E(16, 4, 96)),
            L("latent_attention", A(4, 64, 40, 136, 160, 128, 65, base=250000.0, scaling=(4.0, 128, 16.0, 1.0), kv_from=1), None)],
            streams=4, residual_mult=0.5)
    raise ValueError(variant)


def make(env, cfg, seed=1, max_pos=512, exact=True, tensors=None, **environ):
    old = {k: os.environ.get(k) for k in environ}
    os.environ.update({k: str(v) for k, v in environ.items()})
    try:
        tensors = tensors if tensors is not None else env["synth"].build_madudra(cfg, seed)
        m = env["engine"].StackModel(cfg, max_pos, tensors).load(tensors)
    finally:
        for k, v in old.items():
            if v is None:
                os.environ.pop(k, None)
            else:
                os.environ[k] = v
    m.set_prefill(3 if exact else 1, 1)
    return m, tensors, env["oracle"].MadudraOracle(cfg, tensors)


def dev(env, a):
    return env["engine"].DeviceBuffer.from_numpy(np.ascontiguousarray(a))


def call(env, name, *args):
    env["capi"].check(getattr(env["capi"].lib(), name)(*args, None), name)
    env["capi"].check(env["capi"].lib().tl_device_sync(), "sync")


# ---- each mechanism alone ---------------------------------------------------------------------------------------------
@pytest.mark.parametrize("streams,width,T", [(1, 40, 3), (2, 64, 70), (3, 37, 9), (4, 1028, 20), (5, 48, 30), (16, 12, 5), (3, 2050, 1)])
def test_residual_streams(env, streams, width, T):
    """Write-back of a sublayer into every stream (an unsymmetric mix, so that from and to cannot be swapped), the next
    sublayer's input, its norm, and the sum."""
    orc = env["oracle"]
    rng = np.random.default_rng(streams * width)
    xs = rng.standard_normal((T, streams, width)).astype(np.float32)
    y = rng.standard_normal((T, width)).astype(np.float32)
    mix, a_in, a_out = rng.standard_normal((streams, streams)), rng.standard_normal(streams), rng.standard_normal(streams)
    mix, a_in, a_out = mix.astype(np.float32), a_in.astype(np.float32), a_out.astype(np.float32)
    w, eps, m = rng.standard_normal(width).astype(np.float32), 1e-3, 0.7
    f = lambda a: a.astype(np.float64)
    want = orc.streams_out(f(xs), f(y), f(mix), f(a_out), m)
    xd, yd, md, ind, outd, wd = (dev(env, a) for a in (xs, y, mix, a_in, a_out, w))
    h = env["engine"].DeviceBuffer(4 * T * width)
    sm = env["engine"].DeviceBuffer(4 * T * width)
    call(env, "tl_hyper_connect", xd.ptr, yd.ptr, md.ptr, outd.ptr, m, ind.ptr, wd.ptr, None, eps, h.ptr, sm.ptr, T, streams, width)
    assert np.allclose(xd.to_numpy(np.float32, xs.shape), want, rtol=1e-5, atol=1e-5)
    assert np.allclose(sm.to_numpy(np.float32, y.shape), want.sum(1), rtol=1e-5, atol=2e-5)
    assert np.allclose(h.to_numpy(np.float32, y.shape), orc.layer_norm(orc.streams_in(want, f(a_in)), f(w), eps), rtol=2e-5, atol=2e-5)
    # without a sublayer output the streams stay as they are
    call(env, "tl_hyper_connect", xd.ptr, None, md.ptr, outd.ptr, m, ind.ptr, wd.ptr, None, eps, h.ptr, None, T, streams, width)
    assert np.allclose(xd.to_numpy(np.float32, xs.shape), want, rtol=1e-5, atol=1e-5)


@pytest.mark.parametrize("dim,dims,scaling", [(16, 16, None), (16, 16, (4.0, 64, 8.0, 1.0)), (40, 24, (2.0, 1024, 32.0, 1.0)),
                                              (7, 6, (8.0, 100, 4.0, 2.0)), (2, 2, None), (9, 4, None)])
def test_rotation_of_halves_with_context_extension(env, dim, dims, scaling):
    orc = env["oracle"]
    rng = np.random.default_rng(dim)
    base = 300.0
    x = rng.standard_normal((40, 3, dim)).astype(np.float32)
    sc = dict(zip(("factor", "original", "fast", "slow"), scaling)) if scaling else None
    f, ms = orc.rotary_frequencies(dims, base, sc)
    for start in (0, 7, 4000):
        want = orc.rotate_halves(x.astype(np.float64), np.arange(start, start + 40), dims, f, ms)
        xd = dev(env, x)
        call(env, "tl_rotary_halves", xd.ptr, 40, start, 3, dim, dims, base, *(scaling or (0.0, 0.0, 0.0, 0.0)))
        assert np.allclose(xd.to_numpy(np.float32, x.shape), want, rtol=1e-5, atol=3e-6), start
        if start == 7 and dims > 2:                                # the neighbouring pairing is a different function
            near = want.copy()
            near[..., :dims] = near[..., :dims].reshape(40, 3, dims // 2, 2).swapaxes(-1, -2).reshape(40, 3, dims)
            assert not np.allclose(near, want, atol=1e-2)


@pytest.mark.parametrize("C,taps", [(72, 4), (37, 5), (16, 1), (9, 2), (300, 3)])
def test_convolution_with_an_output_bias(env, C, taps):
    synth, orc = env["synth"], env["oracle"]
    rng = np.random.default_rng(C * taps)
    w = synth.to_bf16(rng.standard_normal((C, taps)).astype(np.float32))
    b = rng.standard_normal(C).astype(np.float32)
    n = 110
    x = rng.standard_normal((n, C)).astype(np.float32)
    want, hist_want = orc.causal_conv(x.astype(np.float64), orc.widen(w), b.astype(np.float64), np.zeros((taps - 1, C)))
    want = orc.silu(want)
    for ld in (C, C + 4, C + 8):                                      # dense rows, and columns of wider rows
        wide = np.full((n, ld), np.nan, np.float32)
        wide[:, :C] = x
        wd, bd, hist = dev(env, w), dev(env, b), dev(env, np.zeros((max(taps - 1, 1), C), np.float32))
        got, p = [], 0
        for size in (1, 2, 70, 3, 1, 33):
            xd = dev(env, wide[p:p + size])
            od = env["engine"].DeviceBuffer(4 * size * C)
            call(env, "tl_causal_conv_bias", xd.ptr, ld, C, taps, size, bd.ptr, wd.ptr, hist.ptr, 1, od.ptr, C)
            got.append(od.to_numpy(np.float32, (size, C)))
            p += size
        assert p == n and np.allclose(np.concatenate(got), want, rtol=1e-5, atol=1e-5)
        if taps > 1:
            assert np.allclose(hist.to_numpy(np.float32, (taps - 1, C)), hist_want, rtol=1e-6, atol=1e-6)


@pytest.mark.parametrize("experts,top,scale", [(12, 3, 2.5), (8, 8, 1.0), (5, 1, 0.3), (130, 6, 1.7), (1, 1, 2.0), (100, 70, 1.0)])
def test_softmax_router(env, experts, top, scale):
    """Weights are the softmax over ALL experts (a token's weights do not sum to one), times the factor."""
    synth, orc = env["synth"], env["oracle"]
    rng = np.random.default_rng(experts + top)
    T, width = 64, 48
    w = synth.to_bf16((rng.standard_normal((experts, width)) * 0.4).astype(np.float32))
    x = rng.standard_normal((T, width)).astype(np.float32)
    z = x.astype(np.float64) @ orc.widen(w).T
    wd, xd = dev(env, w), dev(env, x)
    ids, wts = env["engine"].DeviceBuffer(4 * T * top), env["engine"].DeviceBuffer(4 * T * top)
    call(env, "tl_moe_route_softmax", xd.ptr, T, width, wd.ptr, experts, top, scale, ids.ptr, wts.ptr)
    gi, gw = ids.to_numpy(np.int32, (T, top)), wts.to_numpy(np.float32, (T, top))
    for t in range(T):
        wi, ww = orc.route_softmax(z[t], top, scale)
        assert list(gi[t]) == list(wi), t
        assert np.allclose(gw[t], ww, rtol=1e-5, atol=1e-8)
    assert experts == top or (gw.sum(1) < 0.999 * scale).any()


def test_gelu_of_a_product(env):
    """The exact (erf) form, in the one-token product and in the chunk products' epilogue; far from the tanh form."""
    synth, orc = env["synth"], env["oracle"]
    rng = np.random.default_rng(5)
    rows, cols, T = 70, 40, 100
    w = synth.to_bf16((rng.standard_normal((rows, cols)) * 0.4).astype(np.float32))
    x = rng.standard_normal((T, cols)).astype(np.float32)
    z = x.astype(np.float64) @ orc.widen(w).T
    want = orc.gelu(z)
    tanh_form = 0.5 * z * (1 + np.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))
    assert np.abs(want - tanh_form).max() > 1e-4
    wd = dev(env, w)
    for n, terms in ((1, 0), (T, 3)):
        xd, yd = dev(env, x[:n]), env["engine"].DeviceBuffer(4 * n * rows)
        call(env, "tl_dense_matmul_act", wd.ptr, rows, cols, xd.ptr, yd.ptr, n, terms, 3, 0.0, 0.0, 0)
        assert np.abs(yd.to_numpy(np.float32, (n, rows)) - want[:n]).max() < 1e-5


@pytest.mark.parametrize("T,width,parts", [(5, 48, 1), (70, 96, 8), (3, 37 * 3, 37), (2, 2048, 2), (9, 30, 30)])
def test_norm_in_parts(env, T, width, parts):
    orc = env["oracle"]
    rng = np.random.default_rng(width)
    x = (rng.standard_normal((T, width)) * np.repeat(np.exp(rng.standard_normal(parts)), width // parts)).astype(np.float32)
    w = rng.standard_normal(width).astype(np.float32)
    xd, wd = dev(env, x), dev(env, w)
    call(env, "tl_part_norm", xd.ptr, wd.ptr, T, width, parts, 1e-4, None, None, 0, 0)
    want = orc.rms(x.astype(np.float64).reshape(T, parts, -1), 1e-4).reshape(T, width) * w
    assert np.allclose(xd.to_numpy(np.float32, x.shape), want, rtol=1e-5, atol=1e-6)


SSM_SHAPES = [(6, 3, 20, 12), (1, 1, 1, 1), (4, 2, 64, 64), (3, 1, 5, 7), (4, 1, 128, 40), (2, 1, 130, 48), (2, 2, 300, 33), (2, 1, 33, 65)]


@pytest.mark.parametrize("heads,groups,state,vdim", SSM_SHAPES)
def test_state_space_in_portions(env, heads, groups, state, vdim):
    """Portions of 1, 2, 70, 3, 64, 33 and 150 tokens (cuts inside and at the borders of the blocks of 64) against the oracle's
    recurrence, and the state on the device against the oracle's. Steps from tiny to large: decays from almost 1 to almost 0."""
    orc = env["oracle"]
    rng = np.random.default_rng(heads * state + vdim)
    sizes = (1, 2, 70, 3, 64, 33, 150)
    n, inner = sum(sizes), heads * vdim
    C = inner + 2 * groups * state
    xbc = rng.standard_normal((n, C)).astype(np.float32)
    ld = C + 4 + 3
    z = rng.standard_normal((n, inner)).astype(np.float32)
    dt = (rng.standard_normal((n, heads)) * 2.0 - 1.0).astype(np.float32)
    dtb, alog, D = (rng.standard_normal(heads).astype(np.float32) for _ in range(3))
    f = lambda a: a.astype(np.float64)
    step = orc.softplus(f(dt) + f(dtb))
    x = f(xbc[:, :inner]).reshape(n, heads, vdim)
    B = f(xbc[:, inner:inner + groups * state]).reshape(n, groups, state)
    Cm = f(xbc[:, inner + groups * state:]).reshape(n, groups, state)
    S = np.zeros((heads, state, vdim))
    g = heads // groups
    want = np.stack([orc.state_space(x[:, h], B[:, h // g], Cm[:, h // g], step[:, h], math.exp(alog[h]), float(D[h]), S[h])
                     for h in range(heads)], axis=1).reshape(n, inner) * orc.silu(f(z))
    for dense in (True, False):
        rows = xbc if dense else np.concatenate([xbc, np.full((n, ld - C), np.nan, np.float32)], axis=1)
        sd = dev(env, np.zeros((heads, state, vdim), np.float32))
        bd, ad, dd = dev(env, dtb), dev(env, alog), dev(env, D)
        got, p = [], 0
        for size in sizes:
            xd, td, zd = dev(env, rows[p:p + size]), dev(env, dt[p:p + size]), dev(env, z[p:p + size])
            yd = env["engine"].DeviceBuffer(4 * size * inner)
            call(env, "tl_state_space", xd.ptr, rows.shape[1], td.ptr, heads, bd.ptr, ad.ptr, dd.ptr, zd.ptr, inner, sd.ptr, yd.ptr,
                 size, heads, groups, state, vdim)
            got.append(yd.to_numpy(np.float32, (size, inner)))
            p += size
        assert rel_rms(np.concatenate(got), want) < 1e-5
        assert rel_rms(sd.to_numpy(np.float32, S.shape).reshape(1, -1), S.reshape(1, -1)) < 1e-5


@pytest.mark.parametrize("heads,groups,state,vdim", SSM_SHAPES)
@pytest.mark.parametrize("taps", [1, 2, 4])
def test_state_space_step_with_its_convolution(env, heads, groups, state, vdim, taps):
    """Token by token through the one-token launch and the norm launch that shifts the convolution's history."""
    synth, orc = env["synth"], env["oracle"]
    rng = np.random.default_rng(heads + state * vdim)
    n, inner = 9, heads * vdim
    C = inner + 2 * groups * state
    p = rng.standard_normal((n, inner + C + heads)).astype(np.float32)
    w = synth.to_bf16(rng.standard_normal((C, taps)).astype(np.float32))
    cb = rng.standard_normal(C).astype(np.float32)
    dtb, alog, D = (rng.standard_normal(heads).astype(np.float32) for _ in range(3))
    nw = rng.standard_normal(inner).astype(np.float32)
    f = lambda a: a.astype(np.float64)
    u, hist_want = orc.causal_conv(f(p[:, inner:inner + C]), orc.widen(w), f(cb), np.zeros((taps - 1, C)))
    u = orc.silu(u)
    step = orc.softplus(f(p[:, inner + C:]) + f(dtb))
    S = np.zeros((heads, state, vdim))
    g = heads // groups
    y = np.stack([orc.state_space(u[:, :inner].reshape(n, heads, vdim)[:, h],
                                  u[:, inner:inner + groups * state].reshape(n, groups, state)[:, h // g],
                                  u[:, inner + groups * state:].reshape(n, groups, state)[:, h // g], step[:, h], math.exp(alog[h]),
                                  float(D[h]), S[h]) for h in range(heads)], axis=1).reshape(n, inner)
    want = orc.gated_part_norm(y, f(p[:, :inner]), heads, 1e-5, f(nw))
    sd, hd = dev(env, np.zeros((heads, state, vdim), np.float32)), dev(env, np.zeros((max(taps - 1, 1), C), np.float32))
    wd, cd, bd, ad, dd, nd = (dev(env, a) for a in (w, cb, dtb, alog, D, nw))
    got = []
    for t in range(n):
        pd, yd = dev(env, p[t]), env["engine"].DeviceBuffer(4 * inner)
        call(env, "tl_state_space_step", pd.ptr, wd.ptr, cd.ptr, taps, hd.ptr, bd.ptr, ad.ptr, dd.ptr, sd.ptr, yd.ptr, heads, groups,
             state, vdim)
        call(env, "tl_part_norm", yd.ptr, nd.ptr, 1, inner, heads, 1e-5, hd.ptr if taps > 1 else None, pd.ptr + 4 * inner, taps, C)
        got.append(yd.to_numpy(np.float32, (inner,)))
    assert np.allclose(np.stack(got), want, rtol=2e-4, atol=2e-5)
    assert rel_rms(sd.to_numpy(np.float32, S.shape).reshape(1, -1), S.reshape(1, -1)) < 1e-5
    if taps > 1:
        assert np.allclose(hd.to_numpy(np.float32, (taps - 1, C)), hist_want, rtol=1e-6, atol=1e-6)


def test_state_remembers_and_forgets(env):
    """A value written at token 5 by a large step is read back by the same B at token 385 when the steps in between are almost
    zero; one token with a huge step wipes it. In one call, so that the state crosses the blocks inside the kernel."""
    n, state, vdim = 400, 16, 8
    val = np.arange(1.0, vdim + 1.0)
    for wipe in (False, True):
        xbc = np.zeros((n, vdim + 2 * state), np.float32)
        dt = np.full((n, 1), -30.0, np.float32)                       # softplus(-30) = 1e-13: nothing moves
        dt[5] = 1.0
        xbc[5, :vdim], xbc[5, vdim + 3] = val, 2.0
        xbc[385, vdim + state + 3] = 1.0
        if wipe:
            dt[200] = 100.0                                           # decay exp(-100)
        xd, td, sd = dev(env, xbc), dev(env, dt), dev(env, np.zeros((1, state, vdim), np.float32))
        zero, yd = dev(env, np.zeros(1, np.float32)), env["engine"].DeviceBuffer(4 * n * vdim)
        call(env, "tl_state_space", xd.ptr, xbc.shape[1], td.ptr, 1, zero.ptr, zero.ptr, zero.ptr, None, 0, sd.ptr, yd.ptr, n, 1, 1, state,
             vdim)
        y = yd.to_numpy(np.float32, (n, vdim))
        want = (0.0 if wipe else 1.0) * math.log1p(math.e) * 2.0 * val
        assert np.allclose(y[385], want, rtol=1e-5, atol=1e-6) and np.abs(y[:385]).max() == 0.0, wipe


# ---- whole models -----------------------------------------------------------------------------------------------------
VARIANTS = ["mixed", "odd", "equal", "wide"]


@pytest.mark.parametrize("variant", VARIANTS)
def test_residual_stream_after_every_layer(env, variant):
    cfg = small_config(env["synth"], variant)
    m, _, orc = make(env, cfg, seed=11, TL_NO_GRAPH=1)
    toks = np.random.default_rng(1).integers(0, cfg["vocab"], 90).astype(np.int32)
    res = []
    want = orc.forward(list(toks), res)
    got = m.capture_layers(lambda: m.prefill_rows(toks, 0))
    assert [li for li, _ in got] == list(range(len(cfg["layers"])))
    for (li, a), r in zip(got, res):
        assert rel_rms(a, r) < FP32_TOL, (variant, li, cfg["layers"][li]["type"])
    m.reset_kv()
    assert rel_rms(m.prefill_rows(toks, 0), want) < FP32_TOL
    if variant in ("mixed", "wide"):
        m.set_prefill(1, 1)                                       # bf16 activations in the chunk products
        m.reset_kv()
        assert most_rows(m.prefill_rows(toks, 0), want) < BF16_TOL
    m.free()


@pytest.mark.parametrize("variant", VARIANTS)
def test_prompt_against_token_by_token_decoding(env, variant):
    """The whole prompt in one pass, and the same tokens one by one through the captured decode step (from the very first
    token on), give the same logits at every position."""
    cfg = small_config(env["synth"], variant)
    m, _, orc = make(env, cfg, seed=13)
    assert m.graph_captured()
    n = 180 if variant == "wide" else 80
    toks = np.random.default_rng(2).integers(0, cfg["vocab"], n).astype(np.int32)
    want = orc.forward(list(toks))
    whole = m.prefill_rows(toks, 0)
    m.reset_kv()
    steps = np.stack([m.decode(int(t), i)[0] for i, t in enumerate(toks)])
    assert rel_rms(whole, want) < FP32_TOL and rel_rms(steps, want) < FP32_TOL
    assert rel_rms(steps, whole) < FP32_TOL
    m.free()


@pytest.mark.parametrize("variant,chunk", [("mixed", 512), ("mixed", 16), ("wide", 64), ("wide", 100), ("odd", 5), ("equal", 33)])
def test_portions_of_any_size(env, variant, chunk):
    """A prompt cut into portions (down to two tokens and one) gives the logits of the uncut prompt; `chunk` also cuts long
    portions inside the engine: every cut hands over the states, the convolutions' histories and the latent rows, and portions
    above and below the size at which keys are expanded per head alternate."""
    cfg = small_config(env["synth"], variant)
    m, _, orc = make(env, cfg, seed=17, TL_STACK_CHUNK=chunk)
    n = 400 if variant == "wide" else 160
    toks = np.random.default_rng(3).integers(0, cfg["vocab"], n).astype(np.int32)
    want = orc.forward(list(toks))
    for sizes in ([7, 2, 13, 1, 20, 2, 5, 64, 3], [2] * 20 + [66, 2], [1, 1, 1, 2, 1, 3, 70, 2], [n]):
        m.reset_kv()
        outs, p = [], 0
        for s in sizes + [n]:
            s = min(s, n - p)
            if s <= 0:
                break
            outs.append(m.prefill_rows(toks[p:p + s], p))
            p += s
        assert rel_rms(np.concatenate(outs), want) < FP32_TOL, sizes[:4]
    m.free()


def test_cache_and_state_given_back_and_used_again(env):
    cfg = small_config(env["synth"], "mixed")
    m, _, orc = make(env, cfg, seed=19)
    rng = np.random.default_rng(4)
    a = rng.integers(0, cfg["vocab"], 150).astype(np.int32)
    b = rng.integers(0, cfg["vocab"], 40).astype(np.int32)
    m.prefill_rows(a, 0)
    for i in range(5):
        m.decode(int(a[i]), 150 + i)
    m.reset_kv()
    got = m.prefill_rows(b[:30], 0)
    tail = np.stack([m.decode(int(b[i]), i)[0] for i in range(30, 40)])
    assert rel_rms(np.concatenate([got, tail]), orc.forward(list(b))) < FP32_TOL
    m.free()


@pytest.mark.parametrize("expand", [0, 1, 64])
def test_far_keys_and_window_edges_decide_the_logits(env, expand):
    """Scores sharpened (scale times 6), so that a softmax rests on a few keys anywhere in the window: a fault in a far key or a
    window that is one token off moves the logits by far more than the tolerance. Both forms of latent attention (keys expanded
    per head, and attention over the cached rows) in prompts, portions and decoding past the windows; a layer that borrows the
    cache sees further back than its owner, another one less far."""
    synth = env["synth"]
    A, L = synth.madudra_latent, synth.madudra_layer
    s = 6.0 / math.sqrt(24)
    cfg = synth.madudra_config(64, 97, [
        L("latent_attention", A(4, 16, 8, 16, 32, 32, 37, scale=s), None),
        L("latent_attention", A(2, 16, 8, 24, 24, 32, 130, kv_from=0, scale=s), None),
        L("latent_attention", A(3, 16, 8, 8, 24, 32, 2, kv_from=0, scale=s), None)], streams=2, residual_mult=1.0)
    tensors = synth.build_madudra(cfg, 23)
    m, _, orc = make(env, cfg, tensors=tensors, TL_STACK_LATENT_EXPAND=expand)
    toks = np.random.default_rng(5).integers(0, cfg["vocab"], 330).astype(np.int32)
    want = orc.forward(list(toks))
    got = [m.prefill_rows(toks[:129], 0), m.prefill_rows(toks[129:200], 129), m.prefill_rows(toks[200:230], 200),
           m.prefill_rows(toks[230:232], 230)]
    got += [m.decode(int(toks[i]), i)[0][None] for i in range(232, 330)]
    assert rel_rms(np.concatenate(got), want) < FP32_TOL
    # the oracle with one window one token off differs by orders of magnitude more than the tolerance: the test can see it
    for layer, size in ((0, 36), (0, 38), (1, 129), (2, 3)):
        off = json.loads(json.dumps(cfg))
        off["layers"][layer]["mixer"]["mask"]["size"] = size
        assert rel_rms(env["oracle"].MadudraOracle(off, tensors).forward(list(toks)), want) > 100 * FP32_TOL, layer
    m.free()


@pytest.mark.parametrize("heads", [3, 11])
def test_one_key_just_inside_and_just_outside_the_window(env, heads):
    """Attention over latent rows (one key/value head, keys the whole row, values its first columns): one row with a score far
    above the rest is copied by positions up to window - 1 behind it and not seen one further, in a prompt and for single
    tokens, with the row at the edges of the kernels' 32- and 64-key pieces. Rows outside the window hold NaN."""
    capi, orc = env["capi"], env["oracle"]
    rng = np.random.default_rng(3)
    rank, rd, P = 16, 8, 420
    dim = rank + rd
    for window in (5, 40, 64, 65, 129):
        for star in (0, 31, 63, 64, 200):
            q = np.zeros((P, heads, dim), np.float32)
            q[:, :, 1] = 1.0
            rows = (0.05 * rng.standard_normal((P, dim))).astype(np.float32)
            rows[star, 1] = 40.0
            want = orc.softmax_attention(q.astype(np.float64), np.repeat(rows[:, None].astype(np.float64), heads, 1),
                                         np.repeat(rows[:, None, :rank].astype(np.float64), heads, 1), 1.0, np.arange(P), window)
            inside, outside = star + window - 1, star + window
            assert np.abs(want[inside] - rows[star, :rank]).max() < 1e-4 and abs(want[outside][0, 1]) < 1.0
            for start, T in ((0, P), (inside, 1), (outside, 1), (inside - 1 if inside else 0, 40)):
                kc = rows.copy()
                kc[start + T:] = np.nan
                kc[:max(0, start - window + 1)] = np.nan
                qd, kd = dev(env, q[start:start + T]), dev(env, kc)
                od = env["engine"].DeviceBuffer(4 * T * heads * rank)
                call(env, "tl_window_attention_opts", qd.ptr, heads * dim, 0, kd.ptr, dim, 0, kd.ptr, dim, od.ptr, T, start, heads, 1, dim,
                     rank, window, 1.0, 0.0, None, None, 0, None)
                assert np.allclose(od.to_numpy(np.float32, (T, heads, rank)), want[start:start + T], rtol=1e-5, atol=1e-5), (window, star)


@pytest.mark.parametrize("heads,rank,rd,window", [(32, 512, 64, 300), (8, 16, 8, 0), (40, 128, 40, 65), (70, 260, 4, 1), (9, 64, 700 - 64, 33),
                                                  (16, 40, 20, 1000)])
def test_latent_rows_shared_by_many_heads(env, heads, rank, rd, window):
    """Single tokens and portions of up to four over one row of keys and values for all heads, near the start and far into a
    cache: fewer tiles than splits, splits of several tiles, head tiles that are not full. Rows that a position may not see are
    NaN; one far row dominates for some heads."""
    orc = env["oracle"]
    rng = np.random.default_rng(heads + rank)
    dim, P = rank + rd, 2700
    rows = rng.standard_normal((P, dim)).astype(np.float32)
    scale = 2.0 / math.sqrt(dim)
    for start, T in ((0, 1), (1, 1), (31, 2), (32, 1), (63, 4), (600, 3), (P - 1, 1)):
        q = rng.standard_normal((T, heads, dim)).astype(np.float32)
        kc = rows.copy()
        far = max(0, start - (window or P) + T) if window != 1 else start
        q[:, ::3] = (10.0 * rows[far])[None, None] / np.linalg.norm(rows[far])
        kc[start + T:] = np.nan
        if window > 0:
            kc[:max(0, start - window + 1)] = np.nan
        qd, kd = dev(env, q), dev(env, kc)
        od = env["engine"].DeviceBuffer(4 * T * heads * rank)
        call(env, "tl_window_attention_opts", qd.ptr, heads * dim, 0, kd.ptr, dim, 0, kd.ptr, dim, od.ptr, T, start, heads, 1, dim, rank,
             window, scale, 0.0, None, None, 0, None)
        want = orc.softmax_attention(q.astype(np.float64), np.broadcast_to(rows[:, None], (P, heads, dim)).astype(np.float64),
                                     np.broadcast_to(rows[:, None, :rank], (P, heads, rank)).astype(np.float64), scale,
                                     np.arange(start, start + T), window)
        assert np.allclose(od.to_numpy(np.float32, (T, heads, rank)), want, rtol=3e-5, atol=3e-6), (start, T)


def test_first_tokens_of_a_sequence(env):
    """Positions 0 .. 4, each as a prompt of its own length and as single tokens: zeros before the start in the convolutions,
    empty states, a softmax over one key."""
    cfg = small_config(env["synth"], "mixed")
    m, _, orc = make(env, cfg, seed=41)
    toks = np.array([7, 7, 3, 90, 12], np.int32)
    want = orc.forward(list(toks))
    for n in range(1, 6):
        m.reset_kv()
        assert rel_rms(m.prefill_rows(toks[:n], 0), want[:n]) < FP32_TOL, n
    m.reset_kv()
    steps = np.stack([m.decode(int(t), i)[0] for i, t in enumerate(toks)])
    assert rel_rms(steps, want) < FP32_TOL
    m.free()


def test_long_decoding_and_device_loops(env):
    """Greedy generation on the device (graph replays back to back) equals the oracle's token-by-token arg-max, well past the
    windows; the sampled loop is reproducible by seed and stays inside the vocabulary."""
    cfg = small_config(env["synth"], "mixed")
    m, _, orc = make(env, cfg, seed=29)
    prompt = np.array([3, 14, 15, 92, 65, 35], np.int32)
    want = orc.generate_greedy(list(prompt), 120)
    last_row = np.array([len(prompt) - 1], np.int32)
    first = int(np.argmax(m.prefill_rows(prompt, 0, last_row)[0]))
    assert [first] + list(m.generate_greedy(first, len(prompt), 119)) == want
    runs = []
    for _ in range(2):
        m.reset_kv()
        m.prefill_rows(prompt, 0, last_row)
        runs.append(list(m.generate_sampled(first, len(prompt), 30, temperature=0.9, top_k=20, top_p=0.95, seed=7)))
    assert runs[0] == runs[1] and all(0 <= t < cfg["vocab"] for t in runs[0])
    m.free()


def test_graph_replays_match_the_eager_step(env):
    """The captured decode step, replayed many times with prompt work and synchronisations in between, gives the logits of
    the step enqueued launch by launch."""
    cfg = small_config(env["synth"], "mixed")
    toks = np.random.default_rng(8).integers(0, cfg["vocab"], 60).astype(np.int32)
    tensors = env["synth"].build_madudra(cfg, 37)
    eager, _, _ = make(env, cfg, tensors=tensors, TL_NO_GRAPH=1)
    graph, _, _ = make(env, cfg, tensors=tensors)
    assert graph.graph_captured() and not eager.graph_captured()
    for m in (eager, graph):
        m.prefill_rows(toks[:20], 0, np.array([19], np.int32))
    for i in range(20, 60):
        if i == 40:
            for m in (eager, graph):
                m.prefill_rows(toks[40:42], 40)
        if 40 <= i < 42:
            continue
        a, b = eager.decode(int(toks[i]), i)[0], graph.decode(int(toks[i]), i)[0]
        assert np.array_equal(a, b), i
    eager.free()
    graph.free()


def test_one_token_step_with_and_without_its_fusions(env):
    """The one-token step as it is served against one with the router as a launch of its own, one whose token goes through the
    chunk products and the block walk, and the oracle."""
    cfg = small_config(env["synth"], "mixed")
    toks = np.random.default_rng(9).integers(0, cfg["vocab"], 70).astype(np.int32)
    tensors = env["synth"].build_madudra(cfg, 43)
    served, _, orc = make(env, cfg, tensors=tensors)
    plain, _, _ = make(env, cfg, tensors=tensors, TL_STACK_FUSE_ROUTER=0)
    chunked, _, _ = make(env, cfg, tensors=tensors, TL_STACK_GEMV=0)
    assert served.graph_nodes() < plain.graph_nodes()
    want = orc.forward(list(toks))
    for m in (served, plain, chunked):
        m.prefill_rows(toks[:25], 0, np.array([24], np.int32))
        assert rel_rms(np.stack([m.decode(int(toks[i]), i)[0] for i in range(25, 70)]), want[25:]) < FP32_TOL
        m.free()


def test_generation_through_the_host_session(env, tmp_path):
    """The framework's own entry point: a checkpoint folder opened by tlhost::Session (model registry, config.json reader,
    safetensors loader), greedy generate() for a short and a long prompt, generate_batch over unequal prompts against each
    alone, and the step function a scheduler drives."""
    from tinyllama_cpp_amd import hostapi
    synth = env["synth"]
    cfg = small_config(synth, "mixed")
    tensors = synth.build_madudra(cfg, 31)
    synth.write_stack_dir(str(tmp_path / "ckpt"), cfg, tensors)
    orc = env["oracle"].MadudraOracle(cfg, tensors)
    s = hostapi.Session(str(tmp_path / "ckpt"), 0, 256)
    info = s.info()
    assert info["architecture"] == "Madudra" and info["vocab"] == cfg["vocab"] and info["max_pos"] == 256
    s.set_repetition_penalty(1.0)
    s.set_exact(True)
    rng = np.random.default_rng(6)
    for n in (5, 45):
        prompt = rng.integers(0, cfg["vocab"], n).astype(np.int32)
        assert list(s.generate(prompt, steps=24, temperature=0.0)) == orc.generate_greedy(list(prompt), 24)
    prompts = [rng.integers(0, cfg["vocab"], n).astype(np.int32) for n in (3, 40, 11)]
    s.set_max_batch(3)
    for p, o in zip(prompts, s.generate_batch(prompts, steps=10, temperature=0.0)):
        assert list(o) == orc.generate_greedy(list(p), 10)
    toks = rng.integers(0, cfg["vocab"], 60).astype(np.int32)
    orc.reset()
    want = orc.forward(list(toks))
    s.reset()
    got = [s.forward(toks[:37], 0, [0, 5, 36]), s.forward(toks[37:39], 37, [1])]
    got += [s.forward(toks[i:i + 1], i, [0]) for i in range(39, 60)]
    assert rel_rms(np.concatenate(got), want[[0, 5, 36, 38] + list(range(39, 60))]) < FP32_TOL
    s.close()
    # a layer that borrows a later layer's cache, or one with another rotation, is refused, and so is an unknown layer type
    for name, change, match in (("later", lambda c: c["layers"][2]["mixer"].update(kv_from=4), "kv_from"),
                                ("other", lambda c: c["layers"][2]["mixer"]["rot"].update(base=77.0), "rotation"),
                                ("type", lambda c: c["layers"][0].update(type="mamba3"), "unknown layer type")):
        bad = json.loads(json.dumps(cfg))
        change(bad)
        synth.write_stack_dir(str(tmp_path / name), bad, tensors)
        with pytest.raises(hostapi.TlHostError, match=match):
            hostapi.Session(str(tmp_path / name), 0, 64)


def test_schedule_replayed_by_the_trace_program(env, tmp_path):
    """The command-line program that replays a recorded schedule over a checkpoint folder: a whole prompt, then a second
    request in portions and single tokens after the first one gave its cache and states back; both number formats."""
    import subprocess
    synth = env["synth"]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    exe = os.path.join(root, "tinyllama.cpp_amd", "host", "tl_trace")
    assert os.path.exists(exe), "build the host layer first (make -C tinyllama.cpp_amd/host)"
    cfg = small_config(synth, "mixed")
    tensors = synth.build_madudra(cfg, 53)
    synth.write_stack_dir(str(tmp_path / "ckpt"), cfg, tensors)
    orc = env["oracle"].MadudraOracle(cfg, tensors)
    rng = np.random.default_rng(11)
    a = [int(t) for t in rng.integers(0, cfg["vocab"], 90)]
    b = [int(t) for t in rng.integers(0, cfg["vocab"], 70)]
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a, "want": [0, 1, 40, 89]}], "end": ["a"]},
             {"step": 1, "entries": [{"id": "b", "tokens": b[:37], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[37:39], "want": [0, 1]}], "end": []}]
    steps += [{"step": 3 + i, "entries": [{"id": "b", "tokens": [b[39 + i]], "want": [0]}], "end": ["b"] if 39 + i == 69 else []}
              for i in range(31)]
    want_a = orc.forward(a)[[0, 1, 40, 89]]
    orc.reset()
    want_b = orc.forward(b)[37:]
    for dtype, tol, err in (("float32", FP32_TOL, rel_rms), ("bfloat16", BF16_TOL, most_rows)):
        out = tmp_path / dtype
        out.mkdir()
        r = subprocess.run([exe, "--model", str(tmp_path / "ckpt"), "--dtype", dtype, "--out", str(out), "--max-tokens", "96"],
                           input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
        assert r.returncode == 0, r.stderr
        assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(len(steps))]
        assert not (out / "1.f32").exists()
        got_a = np.fromfile(out / "0.f32", np.float32).reshape(4, cfg["vocab"])
        got_b = np.concatenate([np.fromfile(out / f"{i}.f32", np.float32).reshape(-1, cfg["vocab"]) for i in range(2, len(steps))])
        assert err(got_a, want_a) < tol and err(got_b, want_b) < tol, dtype


def random_config(synth, seed):
    """A configuration drawn at random: layer order, head counts, sizes (also indivisible by 4), windows, shared caches, taps,
    norm parts, groups, routers, streams, with and without feed-forward."""
    rng = np.random.default_rng(5000 + seed)
    A, M, E, L = synth.madudra_latent, synth.madudra_mamba, synth.madudra_moe, synth.madudra_layer
    pick = lambda xs: xs[int(rng.integers(0, len(xs)))]
    layers, owners = [], []
    for i in range(int(rng.integers(2, 7))):
        ml = None
        if rng.random() < 0.75:
            E_n = int(pick([1, 2, 5, 8, 20]))
            ml = E(E_n, int(rng.integers(1, min(E_n, 6) + 1)), int(pick([5, 16, 24, 72])), scale=float(pick([0.5, 1.0, 2.5])))
        if rng.random() < 0.5:
            G = int(pick([1, 2, 3]))
            H, v = G * int(pick([1, 2, 4])), int(pick([3, 8, 20, 64]))
            parts = pick([p for p in (1, 2, 4, G, H) if (H * v) % p == 0])
            layers.append(L("mamba2", M(H, v, int(pick([3, 8, 16, 64, 130, 200])), groups=G, conv=int(pick([1, 2, 4, 6])), norm_groups=parts), ml))
            continue
        share = owners and rng.random() < 0.5
        if share:
            j = pick(owners)
            o = layers[j]["mixer"]
            rd, rk, base, sc = o["rot_dim"], o["kv_rank"], o["rot"]["base"], o["rot"].get("scaling")
            sc = tuple(sc[k] for k in ("factor", "original", "fast", "slow")) if sc else None
        else:
            j, rd, rk, base = None, int(pick([2, 6, 8, 16])), int(pick([5, 16, 40, 64])), float(pick([100.0, 10000.0, 500000.0]))
            sc = pick([None, (2.0, 64, 8.0, 1.0), (8.0, 256, 32.0, 1.0), (1.5, 100, 2.0, 1.0)])
            owners.append(i)
        d = int(pick([5, 8, 16, 48]))
        layers.append(L("latent_attention", A(int(pick([1, 2, 3, 6])), d, rd, int(pick([3, 8, 16, 40])), int(pick([7, 16, 40])), rk,
                                              int(pick([0, 1, 2, 7, 33, 64, 100])), base=base, scaling=sc, kv_from=j,
                                              scale=float(pick([0.1, (d + rd) ** -0.5, 0.4]))), ml))
    return synth.madudra_config(int(pick([24, 50, 64, 100])), int(pick([40, 97, 130])), layers, streams=int(pick([1, 2, 3, 4, 6])),
                                residual_mult=float(pick([0.3, 0.5, 1.0, 1.4])), eps=float(pick([1e-6, 1e-5, 1e-2])),
                                embed_scale=float(pick([0.5, 1.0, 3.0, 8.0])))


@pytest.mark.parametrize("seed", range(16))
def test_configurations_drawn_at_random(env, seed, tmp_path):
    """Through the host session over a checkpoint folder (so the configuration reader is part of what is tested): a prompt in
    portions and decoded tokens against the oracle, twice over so that state and cache are given back in between."""
    from tinyllama_cpp_amd import hostapi
    synth = env["synth"]
    cfg = random_config(synth, seed)
    tensors = synth.build_madudra(cfg, seed)
    synth.write_stack_dir(str(tmp_path / "ckpt"), cfg, tensors)
    orc = env["oracle"].MadudraOracle(cfg, tensors)
    rng = np.random.default_rng(seed)
    n = 200
    s = hostapi.Session(str(tmp_path / "ckpt"), 0, n)
    s.set_exact(True)
    for _ in range(2):
        toks = rng.integers(0, cfg["vocab"], n).astype(np.int32)
        orc.reset()
        want = orc.forward(list(toks))
        s.reset()
        got, p = [], 0
        for size in [int(x) for x in rng.integers(1, 24, 5)] + [2, 66]:
            got.append(s.forward(toks[p:p + size], p, list(range(size))))
            p += size
        got += [s.forward(toks[i:i + 1], i, [0]) for i in range(p, n)]
        # (drawn sizes include norms over three channels, which magnify the last bits of single rows)
        assert rel_rms(np.concatenate(got), want) < 4 * FP32_TOL, json.dumps(cfg)
    s.close()
