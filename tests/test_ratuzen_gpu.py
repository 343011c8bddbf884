"""Ratuzen layer-list models on the GPU against the plain float64 implementation in oracle/ratuzen_oracle.py.

Every test builds its own small configuration and random weights (synth.build_ratuzen). The product path is libtlhip.so
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


@pytest.fixture(scope="module")
def env(pkg):
    from tinyllama_cpp_amd import capi, engine, synth
    from oracle import ratuzen_oracle
    engine.init(0)
    return {"capi": capi, "engine": engine, "synth": synth, "oracle": ratuzen_oracle}


def small_config(synth, variant="mixed"):
    K, C, D, L = synth.ratuzen_chunked, synth.ratuzen_causal, synth.ratuzen_delta, synth.ratuzen_layer
    if variant == "mixed":  # unequal layers, grouped heads, a layer without feed-forward
        return synth.ratuzen_config(72, 101, [
            L("parallel", K(6, 3, 16, 12, 11, 3, 12, 20, [0.5, 0.97, 1.0], rot_dims=8, scaling=(8.0, 1.0, 4.0, 64)), 56),
            L("delta", D(4, 2, 12, 20, conv=3), 40),
            L("parallel_2", C(6, 2, 16, 12, 2, 24, 8, tau=8.0, rot_dims=12, factor=3.0), 48),
            L("parallel", K(4, 1, 20, 28, 50, 1, 8, 36, [0.99], base=500.0), None),
            L("delta", D(2, 1, 24, 8, conv=2), None),
            L("parallel_2", C(4, 4, 8, 16, 3, 16, 12, tau=16.0), 24)])
    if variant == "odd":  # nothing divisible by 4: every scalar fallback path
        return synth.ratuzen_config(37, 53, [
            L("parallel_2", C(3, 1, 10, 7, 3, 5, 9, tau=2.5, rot_dims=6, factor=1.5), 9),
            L("parallel", K(3, 3, 6, 5, 9, 1, 7, 11, [0.8], rot_dims=4, scaling=(3.0, 1.0, 2.0, 20)), 11),
            L("delta", D(3, 3, 5, 7, conv=5), 7)], eps=1e-3, logit_scale=0.5)
    if variant == "equal":  # values a model may happen to make equal or 1
        return synth.ratuzen_config(32, 64, [
            L("parallel", K(1, 1, 32, 32, 1, 1, 32, 32, [1.0], scale=1.0), 32),
            L("delta", D(1, 1, 32, 32, conv=1), 32),
            L("parallel_2", C(1, 1, 32, 32, 1, 32, 32, tau=1.0, factor=1.0, scale=1.0), 32),
            L("parallel", K(2, 2, 16, 16, 0, 2, 16, 16, [0.0, 0.0], scaling=(1.0, 1.0, 4.0, 64)), 16),
            L("parallel_2", C(2, 2, 16, 16, 2, 2, 2), 16)], logit_scale=1.0)
    if variant == "wide":  # several tiles in every product, sizes past the kernels' register-resident limits
        return synth.ratuzen_config(320, 300, [
            L("parallel_2", C(8, 2, 64, 64, 4, 96, 64, rot_dims=32, factor=4.0), 384),
            L("parallel", K(8, 4, 40, 72, 130, 4, 160, 48, [0.3, 0.9, 0.99, 0.9995], scaling=(4.0, 1.0, 4.0, 256)), 160),
            L("delta", D(4, 2, 96, 64, conv=4), 200),
            L("parallel", K(4, 4, 136, 40, 64, 2, 64, 136, [0.95, 0.6], rot_dims=64), 96),
            L("parallel_2", C(4, 2, 136, 40, 2, 130, 136, tau=4.0), 64)], logit_scale=2.5)
    raise ValueError(variant)


def make(env, cfg, seed=1, max_pos=512, exact=True, tensors=None, **environ):
    old = {k: os.environ.get(k) for k in environ}
    os.environ.update({k: str(v) for k, v in environ.items()})
    try:
        tensors = tensors if tensors is not None else env["synth"].build_ratuzen(cfg, seed)
        m = env["engine"].StackModel(cfg, max_pos, tensors).load(tensors)
    finally:
        for k, v in old.items():
            if v is None:
                os.environ.pop(k, None)
            else:
                os.environ[k] = v
    m.set_prefill(3 if exact else 1, 1)
    return m, tensors, env["oracle"].RatuzenOracle(cfg, tensors)


def dev(env, a):
    return env["engine"].DeviceBuffer.from_numpy(np.ascontiguousarray(a))


def sync(env):
    env["capi"].check(env["capi"].lib().tl_device_sync(), "sync")


def f64(a):
    return np.asarray(a, np.float64)


# ---- each mechanism alone ---------------------------------------------------------------------------------------------
@pytest.mark.parametrize("heads,dim,rot_dims,halves,norm,scaling", [
    (5, 16, 16, 0, 0, None), (5, 16, 8, 1, 1, None), (3, 20, 12, 0, 1, ("linear", 3.0)), (4, 64, 64, 1, 1, ("linear", 4.0)),
    (2, 130, 96, 1, 0, ("wave", 8.0, 1.0, 4.0, 128)), (3, 48, 32, 0, 0, ("wave", 4.0, 1.0, 4.0, 1000)), (1, 7, 4, 1, 1, ("wave", 2.0, 2.0, 3.0, 40)),
    (2, 512, 512, 1, 1, ("linear", 2.0)), (3, 9, 0, 0, 1, None)])
def test_head_norm_rotation_and_frequency_scaling(env, heads, dim, rot_dims, halves, norm, scaling):
    """Near the start and far out (where an angle that is off by a rounding of the frequency would show), for one token and many."""
    capi, orc = env["capi"], env["oracle"]
    rng = np.random.default_rng(dim + rot_dims)
    rot = {"base": 700.0, "dims": rot_dims}
    kind, factor, original, fast, slow = 0, 0.0, 0.0, 0.0, 0.0
    if scaling and scaling[0] == "linear":
        rot["scaling"] = {"factor": scaling[1]}
        kind, factor = 1, scaling[1]
    elif scaling:
        rot["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling[1:]))
        kind, factor, slow, fast, original = 2, *scaling[1:]
    w = (1.0 + 0.4 * rng.standard_normal(dim)).astype(np.float32)
    wd = dev(env, w)
    for start, T in ((0, 9), (3900, 5), (17, 1)):
        x = rng.standard_normal((T, heads, dim)).astype(np.float32)
        xd = dev(env, x)
        capi.check(capi.lib().tl_rotary_normed(xd.ptr, T, start, heads, dim, rot_dims, 700.0, kind, factor, original, fast, slow, halves,
                                               wd.ptr if norm else None, 1e-5, None), "tl_rotary_normed")
        sync(env)
        want = f64(x)
        if norm:
            want = orc.rms(want, 1e-5) * f64(w)
        if rot_dims:
            want = orc.rotate(want, np.arange(start, start + T), orc.frequencies(rot), bool(halves))
        assert np.allclose(xd.to_numpy(np.float32, (T, heads, dim)), want, rtol=1e-5, atol=3e-6), (start, T)


def test_wavelength_scaling_uses_all_three_ranges(env):
    """The frequencies of the tests above cover pairs that stay, pairs that are divided and pairs in between."""
    orc = env["oracle"]
    for dims, sc in ((96, dict(factor=8.0, low=1.0, high=4.0, original=128)), (32, dict(factor=4.0, low=1.0, high=4.0, original=1000))):
        f0 = orc.frequencies({"base": 700.0, "dims": dims})
        r = orc.frequencies({"base": 700.0, "dims": dims, "scaling": sc}) / f0
        assert (r == 1.0).any() and np.isclose(r, 1.0 / sc["factor"]).any() and ((r < 0.999) & (r > 1.001 / sc["factor"])).any()


def run_chunk_attention(env, q, kc, vc, start, chunk, scale, gate=None):
    capi = env["capi"]
    T, heads, dim, vdim, kv_heads = q.shape[0], q.shape[1], q.shape[2], vc.shape[2], kc.shape[1]
    qd, kd, vd = dev(env, q), dev(env, kc), dev(env, vc)
    gd = dev(env, gate) if gate is not None else None
    od = env["engine"].DeviceBuffer(4 * T * heads * vdim)
    capi.check(capi.lib().tl_chunk_attention(qd.ptr, kd.ptr, vd.ptr, od.ptr, T, start, heads, kv_heads, dim, vdim, chunk, scale,
                                             gd.ptr if gd else None, gate.shape[1] if gate is not None else 0, None), "attention")
    sync(env)
    return od.to_numpy(np.float32, (T, heads, vdim))


@pytest.mark.parametrize("heads,kv_heads,dim,vdim,chunk", [(6, 3, 8, 12, 11), (3, 1, 10, 7, 64), (4, 2, 64, 64, 130), (2, 1, 136, 40, 33),
                                                          (4, 4, 48, 48, 0), (2, 1, 16, 16, 1), (8, 1, 32, 130, 256)])
def test_chunked_attention_with_gate_over_poisoned_caches(env, heads, kv_heads, dim, vdim, chunk):
    """Prompts (the matrix-core kernel), short portions and single tokens far into a cache (key splits). Cache rows that no position
    of the call may see -- behind it, or before its chunk -- hold NaN."""
    orc = env["oracle"]
    rng = np.random.default_rng(dim + chunk)
    P = 700
    k = rng.standard_normal((P, kv_heads, dim)).astype(np.float32)
    v = rng.standard_normal((P, kv_heads, vdim)).astype(np.float32)
    scale = 2.0 / math.sqrt(dim)
    for start, T in ((0, 130), (0, 1), (1, 1), (63, 3), (64, 1), (300, 40), (699, 1), (640, 60), (511, 2)):
        q = rng.standard_normal((T, heads, dim)).astype(np.float32)
        gate = (2.0 * rng.standard_normal((T, heads + 3))).astype(np.float32) if T % 2 else None
        kc, vc = k.copy(), v.copy()
        lo = orc.first_visible(start, chunk)
        kc[start + T:], vc[start + T:], kc[:lo], vc[:lo] = np.nan, np.nan, np.nan, np.nan
        got = run_chunk_attention(env, q, kc, vc, start, chunk, scale, gate)
        want = orc.softmax_attention(f64(q), f64(k), f64(v), scale, np.arange(start, start + T), chunk)
        if gate is not None:
            want = want * orc.sigmoid(f64(gate[:, :heads]))[:, :, None]
        assert np.allclose(got, want, rtol=3e-5, atol=3e-6), (start, T)


def test_a_key_at_either_end_of_its_chunk(env):
    """One key with a score far above the rest, as the first and as the last position of a chunk: every later position of the same
    chunk copies its value, the first position of the next chunk does not see it, nor does anything before it. In a prompt and for
    single tokens, for chunks that start inside and at the edges of the kernels' 32- and 64-key pieces."""
    orc = env["oracle"]
    rng = np.random.default_rng(3)
    dim, vdim, P = 16, 8, 420
    for chunk in (5, 32, 40, 64, 65, 129):
        for star in (chunk, 2 * chunk - 1, 2 * chunk, 3 * chunk - 2):
            if star + 1 >= P:
                continue
            end = (star // chunk + 1) * chunk                      # first position that does not see it any more
            q = np.zeros((P, 1, dim), np.float32)
            q[:, 0, 0] = 1.0
            k = (0.01 * rng.standard_normal((P, 1, dim))).astype(np.float32)
            k[star, 0, 0] = 30.0
            v = rng.standard_normal((P, 1, vdim)).astype(np.float32)
            want = orc.softmax_attention(f64(q), f64(k), f64(v), 1.0, np.arange(P), chunk)
            assert np.abs(want[star:min(end, P)] - v[star]).max() < 1e-6
            if end < P:
                assert np.abs(want[end] - v[star]).max() > 1e-2
            got = run_chunk_attention(env, q, k, v, 0, chunk, 1.0)
            assert np.allclose(got, want, rtol=1e-5, atol=1e-6), (chunk, star)
            for i in (star, end - 1, end):
                if i < P:
                    one = run_chunk_attention(env, q[i:i + 1], k, v, i, chunk, 1.0)
                    assert np.allclose(one[0], want[i], rtol=1e-5, atol=1e-6), (chunk, star, i)


@pytest.mark.parametrize("rows,cols,act,lo,hi", [(50, 24, 4, 13, 37), (300, 40, 4, 128, 300), (37, 9, 5, 0, 0), (260, 256, 0, 0, 0), (64, 16, 5, 0, 64)])
def test_product_with_bias_and_activation_range(env, rows, cols, act, lo, hi):
    """silu or sigmoid^P on a range of the output features, a bias on all of them; the one-token product and both chunk products."""
    capi, synth, orc = env["capi"], env["synth"], env["oracle"]
    rng = np.random.default_rng(rows)
    w = synth.to_bf16((rng.standard_normal((rows, cols)) * 2.0 / math.sqrt(cols)).astype(np.float32))
    b = rng.standard_normal(rows).astype(np.float32)
    power = 1.0 / 16.0
    wd, bd = dev(env, w), dev(env, b)
    for T, terms in ((1, 0), (70, 3), (70, 1), (150, 3)):
        x = rng.standard_normal((T, cols)).astype(np.float32)
        z = f64(x) @ orc.widen(w).T + f64(b)
        want = z.copy()
        span = slice(lo, hi if hi > 0 else rows)
        if act == 4:
            want[:, span] = orc.silu(z[:, span])
        elif act == 5:
            want[:, span] = orc.sigmoid(z[:, span]) ** power
        xd = dev(env, x)
        od = env["engine"].DeviceBuffer(4 * T * rows)
        capi.check(capi.lib().tl_dense_matmul_bias(wd.ptr, rows, cols, xd.ptr, od.ptr, T, terms, bd.ptr, act, power, 0.0, lo, hi, None), "product")
        sync(env)
        got = od.to_numpy(np.float32, (T, rows))
        assert np.allclose(got, want, rtol=2e-5 if terms != 1 else 3e-2, atol=2e-6 if terms != 1 else 4e-2), (T, terms)


def test_sigmoid_power_keeps_far_tails(env):
    """alpha = sigmoid(z)^(1 / tau) where sigmoid itself would round to 0 or 1: z down to -60 and up to +30."""
    capi, synth = env["capi"], env["synth"]
    z = np.array([-60.0, -20.0, -5.0, 0.0, 5.0, 12.0, 30.0])
    w = synth.to_bf16(np.zeros((len(z), 8), np.float32))
    wd, bd, xd = dev(env, w), dev(env, z.astype(np.float32)), dev(env, np.ones((1, 8), np.float32))
    od = env["engine"].DeviceBuffer(4 * len(z))
    capi.check(capi.lib().tl_dense_matmul_bias(wd.ptr, len(z), 8, xd.ptr, od.ptr, 1, 0, bd.ptr, 5, 1.0 / 16.0, 0.0, 0, 0, None), "product")
    sync(env)
    want = np.exp(-np.logaddexp(0.0, -z) / 16.0)
    assert np.allclose(od.to_numpy(np.float32, (len(z),)), want, rtol=1e-6)


@pytest.mark.parametrize("heads,dim,vdim", [(3, 12, 20), (1, 1, 1), (2, 130, 48), (4, 64, 64), (3, 5, 9)])
def test_channel_decay_recurrence_in_portions(env, heads, dim, vdim):
    """Portions of 1, 2, 40 and 3 tokens against the oracle's recurrence, and the state on the device against the oracle's."""
    capi, orc = env["capi"], env["oracle"]
    rng = np.random.default_rng(heads * dim)
    n, hd = 75, heads * dim
    ld = 2 * hd + heads * vdim + 3
    p = rng.standard_normal((n, ld)).astype(np.float32)
    alpha = (rng.uniform(0.0, 1.0, (n, hd)) ** (1.0 / 16.0)).astype(np.float32)
    part = lambda off, d: f64(p[:, off:off + heads * d]).reshape(n, heads, d)
    q, k, v = part(1, dim), part(1 + hd, dim), part(1 + 2 * hd, vdim)
    S = np.zeros((heads, dim, vdim))
    want = np.stack([orc.linear_recurrence(0.3 * q[:, h], k[:, h], v[:, h], f64(alpha).reshape(n, heads, dim)[:, h], S[h]) for h in range(heads)], axis=1)
    state = dev(env, np.zeros((heads, vdim, dim), np.float32))
    got, at = [], 0
    for size in (1, 2, 40, 3, 1, 28):
        pd, ad = dev(env, p[at:at + size]), dev(env, alpha[at:at + size])
        od = env["engine"].DeviceBuffer(4 * size * heads * vdim)
        capi.check(capi.lib().tl_channel_decay_attention(pd.ptr, ld, 1, 1 + hd, 1 + 2 * hd, ad.ptr, 0.3, state.ptr, od.ptr, size, heads, dim, vdim,
                                                         None), "tl_channel_decay_attention")
        sync(env)
        got.append(od.to_numpy(np.float32, (size, heads, vdim)))
        at += size
    assert at == n and np.allclose(np.concatenate(got), want, rtol=3e-5, atol=1e-5)
    assert np.allclose(state.to_numpy(np.float32, (heads, vdim, dim)).transpose(0, 2, 1), S, rtol=3e-5, atol=1e-5)


@pytest.mark.parametrize("heads,dim,vdim,rank", [(3, 12, 20, 8), (1, 1, 1, 1), (2, 130, 48, 5), (4, 64, 64, 16), (3, 5, 9, 3), (2, 128, 128, 16),
                                                 (2, 32, 200, 40), (1, 256, 512, 64), (2, 16, 70, 2)])
def test_channel_decay_step(env, heads, dim, vdim, rank):
    """The one-token launch (decay projection, recurrence, head norm, gate) over several tokens, output and state."""
    capi, synth, orc = env["capi"], env["synth"], env["oracle"]
    rng = np.random.default_rng(heads + dim + vdim)
    hd, vd, n, tau, eps = heads * dim, heads * vdim, 6, 8.0, 1e-5
    p = rng.standard_normal((n, 2 * hd + 2 * vd + rank)).astype(np.float32)
    a2 = synth.to_bf16((rng.standard_normal((hd, rank)) * 2.0 / math.sqrt(rank)).astype(np.float32))
    b = rng.standard_normal(hd).astype(np.float32)
    w = (1.0 + 0.2 * rng.standard_normal(vdim)).astype(np.float32)
    z = f64(p[:, 2 * hd + 2 * vd:]) @ orc.widen(a2).T + f64(b)
    alpha = (orc.sigmoid(z) ** (1.0 / tau)).reshape(n, heads, dim)
    q, k = f64(p[:, :hd]).reshape(n, heads, dim) * dim ** -0.5, f64(p[:, hd:2 * hd]).reshape(n, heads, dim)
    v, gate = f64(p[:, 2 * hd:2 * hd + vd]).reshape(n, heads, vdim), f64(p[:, 2 * hd + vd:2 * hd + 2 * vd])
    S0 = rng.standard_normal((heads, dim, vdim)).astype(np.float32)
    S = f64(S0)
    o = np.stack([orc.linear_recurrence(q[:, h], k[:, h], v[:, h], alpha[:, h], S[h]) for h in range(heads)], axis=1)
    want = (orc.rms(o, eps) * f64(w)).reshape(n, vd) * orc.silu(gate)
    state, ad, bd, wd = dev(env, S0.transpose(0, 2, 1)), dev(env, a2), dev(env, b), dev(env, w)
    for t in range(n):
        pd = dev(env, p[t])
        od = env["engine"].DeviceBuffer(4 * vd)
        capi.check(capi.lib().tl_channel_decay_step(pd.ptr, ad.ptr, bd.ptr, rank, 1.0 / tau, dim ** -0.5, wd.ptr, eps, state.ptr, od.ptr, heads, dim,
                                                    vdim, None), "tl_channel_decay_step")
        sync(env)
        assert np.allclose(od.to_numpy(np.float32, (vd,)), want[t], rtol=2e-4, atol=2e-5), t
    assert np.allclose(state.to_numpy(np.float32, (heads, vdim, dim)).transpose(0, 2, 1), S, rtol=3e-5, atol=1e-5)


@pytest.mark.parametrize("heads,dim,vdim", [(3, 12, 20), (1, 1, 1), (2, 130, 48), (4, 64, 64), (3, 5, 9), (2, 300, 40), (2, 32, 96)])
def test_constant_decay_recurrence_in_portions(env, heads, dim, vdim):
    """Blocks of the matrix-core walk and the one-token step in turn, portions around the block size of 64; decays from 0 to 1."""
    capi, orc = env["capi"], env["oracle"]
    rng = np.random.default_rng(heads * dim)
    decay = np.array([0.999, 0.6, 1.0, 0.0])[:heads] if dim != 64 else np.array([0.0, 1e-3, 0.9, 1.0])[:heads]
    logd = np.maximum(np.log(np.maximum(decay, 1e-300)), -1e4)
    sizes = (1, 2, 64, 63, 65, 1, 130, 3, 128, 43)
    n, off = sum(sizes), 4
    ld = off + heads * (2 * dim + vdim)
    p = (rng.standard_normal((n, ld)) * 0.5).astype(np.float32)
    v = f64(p[:, off:off + heads * vdim]).reshape(n, heads, vdim)
    k = f64(p[:, off + heads * vdim:off + heads * (vdim + dim)]).reshape(n, heads, dim)
    q = f64(p[:, off + heads * (vdim + dim):]).reshape(n, heads, dim)
    S = np.zeros((heads, dim, vdim))
    want = np.stack([orc.linear_recurrence(q[:, h], k[:, h], v[:, h], decay[h], S[h]) for h in range(heads)], axis=1)
    state, dd = dev(env, np.zeros((heads, dim, vdim), np.float32)), dev(env, logd)
    got, at = [], 0
    for size in sizes:
        pd = dev(env, p[at:at + size])
        od = env["engine"].DeviceBuffer(4 * size * heads * vdim)
        capi.check(capi.lib().tl_constant_decay_attention(pd.ptr + 4 * off, ld, dd.ptr, state.ptr, od.ptr, size, heads, dim, vdim, None), "lightning")
        sync(env)
        got.append(od.to_numpy(np.float32, (size, heads, vdim)))
        at += size
    got = np.concatenate(got)
    for h in range(heads):
        assert np.allclose(got[:, h], want[:, h], rtol=3e-5, atol=2e-6 * np.abs(want[:, h]).max() + 1e-6), h
        assert np.allclose(state.to_numpy(np.float32, (heads, dim, vdim))[h], S[h], rtol=3e-5, atol=2e-6 * np.abs(S[h]).max() + 1e-6), h


def test_constant_decay_remembers_a_far_token(env):
    """One write at position 5, read 380 positions later through whole blocks, a ragged portion and single tokens: decay^380 of it."""
    capi = env["capi"]
    dim, vdim, n = 8, 4, 400
    for decay in (1.0, 0.99):
        p = np.zeros((n, vdim + 2 * dim), np.float32)
        p[5, :vdim] = [1.0, -2.0, 3.0, 0.5]
        p[5, vdim] = 2.0
        p[385, vdim + dim] = 3.0
        state, dd = dev(env, np.zeros((1, dim, vdim), np.float32)), dev(env, np.array([math.log(decay)]))
        got, at = [], 0
        for size in [128, 1, 1, 77, 150, 2] + [1] * 41:
            pd = dev(env, p[at:at + size])
            od = env["engine"].DeviceBuffer(4 * size * vdim)
            capi.check(capi.lib().tl_constant_decay_attention(pd.ptr, vdim + 2 * dim, dd.ptr, state.ptr, od.ptr, size, 1, dim, vdim, None), "lightning")
            sync(env)
            got.append(od.to_numpy(np.float32, (size, vdim)))
            at += size
        got = np.concatenate(got)
        assert at == n and np.allclose(got[385], 6.0 * decay ** 380 * np.array([1.0, -2.0, 3.0, 0.5]), rtol=2e-4)
        assert np.abs(np.delete(got, 385, 0)).max() == 0.0


@pytest.mark.parametrize("T,width", [(1, 96), (5, 37), (70, 320), (1, 1), (3, 5000)])
def test_row_norm_with_gate(env, T, width):
    capi, orc = env["capi"], env["oracle"]
    rng = np.random.default_rng(width)
    x = (3.0 * rng.standard_normal((T, width))).astype(np.float32)
    g = rng.standard_normal((T, width + 2)).astype(np.float32)
    w = (1.0 + 0.3 * rng.standard_normal(width)).astype(np.float32)
    xd, gd, wd = dev(env, x), dev(env, g), dev(env, w)
    capi.check(capi.lib().tl_gated_row_norm(xd.ptr, wd.ptr, gd.ptr, width + 2, T, width, 1e-4, None), "tl_gated_row_norm")
    sync(env)
    want = orc.rms(f64(x), 1e-4) * f64(w) * orc.sigmoid(f64(g[:, :width]))
    assert np.allclose(xd.to_numpy(np.float32, (T, width)), want, rtol=1e-5, atol=1e-6)


@pytest.mark.parametrize("T,width", [(1, 72), (9, 37), (40, 320), (3, 1), (1, 4096), (12, 4096), (2, 16384), (20, 5001)])
def test_two_outputs_join_the_residual_behind_norms_of_their_own(env, T, width):
    """x += 1/2 N(a) + 1/2 N(b) + c and both norms of the new x; then each part left out in turn."""
    capi, orc = env["capi"], env["oracle"]
    rng = np.random.default_rng(width + T)
    mk = lambda s=1.0: (s * rng.standard_normal((T, width))).astype(np.float32)
    vec = lambda: (1.0 + 0.3 * rng.standard_normal(width)).astype(np.float32)
    x, a, b, c, eps = mk(), mk(20.0), mk(0.1), mk(), 1e-5
    aw, bw, w1, w2 = vec(), vec(), vec(), vec()
    for skip in ("", "aw", "bw", "b", "c", "w1", "w2", "abc", "w1w2"):
        use = lambda n: not (skip == n or skip == "abc" and n in ("a", "b", "c") or skip == "w1w2" and n in ("w1", "w2"))
        xd, h1, h2 = dev(env, x), dev(env, np.full((T, width), 7.0, np.float32)), dev(env, np.full((T, width), 7.0, np.float32))
        bufs = {n: dev(env, v) for n, v in (("a", a), ("b", b), ("c", c), ("aw", aw), ("bw", bw), ("w1", w1), ("w2", w2))}
        ua, ub = use("a"), use("b")
        p = lambda n, ok=True: bufs[n].ptr if ok and use(n) else None
        capi.check(capi.lib().tl_resid_two_norms(xd.ptr, p("a"), 0.5, p("aw", ua), p("b"), 0.25, p("bw", ub), p("c"), p("w1"), h1.ptr, p("w2"), h2.ptr,
                                                 T, width, eps, None), "tl_resid_two_norms")
        sync(env)
        want = f64(x)
        if ua:
            want = want + 0.5 * (orc.rms(f64(a), eps) * f64(aw) if use("aw") else f64(a))
        if ub:
            want = want + 0.25 * (orc.rms(f64(b), eps) * f64(bw) if use("bw") else f64(b))
        if use("c"):
            want = want + f64(c)
        assert np.allclose(xd.to_numpy(np.float32, (T, width)), want, rtol=1e-5, atol=2e-6), skip
        for n, h, w in (("w1", h1, w1), ("w2", h2, w2)):
            ref = orc.rms(want, eps) * f64(w) if use(n) else np.full((T, width), 7.0)
            assert np.allclose(h.to_numpy(np.float32, (T, width)), ref, rtol=2e-5, atol=3e-6), (skip, n)


# ---- whole models -----------------------------------------------------------------------------------------------------
VARIANTS = ["mixed", "odd", "equal", "wide"]


@pytest.mark.parametrize("variant", VARIANTS)
def test_residual_stream_after_every_layer(env, variant):
    cfg = small_config(env["synth"], variant)
    m, _, orc = make(env, cfg, seed=11, TL_NO_GRAPH=1)
    rng = np.random.default_rng(1)
    toks = rng.integers(0, cfg["vocab"], 90).astype(np.int32)
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
        got = f64(m.prefill_rows(toks, 0))
        err = np.sqrt(((got - want) ** 2).mean(-1)) / np.sqrt((want * want).mean())
        assert err.max() < BF16_TOL, err
    m.free()


def test_first_token_of_a_long_prompt_keeps_more_bits_in_bf16_mode(env):
    """A recurrence's first read-out is v (k . q), normed: where k . q is small its sign hangs on the last bits of the layer's input.
    So a sequence's first token keeps 16 bits of its activations where the chunk products round them to 8."""
    cfg = small_config(env["synth"], "wide")
    m, tensors, orc = make(env, cfg, seed=3, exact=False)
    loose, _, _ = make(env, cfg, tensors=tensors, exact=False, TL_STACK_EXACT_FIRST=0)
    rng = np.random.default_rng(12)
    worst = [0.0, 0.0]
    for _ in range(12):
        toks = rng.integers(0, cfg["vocab"], 80).astype(np.int32)
        orc.reset()
        want = orc.forward(list(toks[:3]))
        for j, mm in enumerate((m, loose)):
            mm.reset_kv()
            worst[j] = max(worst[j], rel_rms(mm.prefill_rows(toks, 0, np.array([0, 79], np.int32))[:1], want[:1]))
    print(worst)
    assert worst[0] < 1e-3 and worst[1] > 5 * worst[0], worst
    m.free()
    loose.free()


@pytest.mark.parametrize("variant", VARIANTS)
def test_prompt_against_token_by_token_decoding(env, variant):
    """The whole prompt in one pass, and the same tokens one by one through the captured decode step (from the very first
    token on), give the same logits at every position."""
    cfg = small_config(env["synth"], variant)
    m, _, orc = make(env, cfg, seed=13)
    assert m.graph_captured()
    rng = np.random.default_rng(2)
    n = 180 if variant == "wide" else 80
    toks = rng.integers(0, cfg["vocab"], n).astype(np.int32)
    want = orc.forward(list(toks))
    whole = m.prefill_rows(toks, 0)
    m.reset_kv()
    steps = np.stack([m.decode(int(t), i)[0] for i, t in enumerate(toks)])
    assert rel_rms(whole, want) < FP32_TOL and rel_rms(steps, want) < FP32_TOL
    assert rel_rms(steps, whole) < FP32_TOL
    m.free()


@pytest.mark.parametrize("variant,chunk", [("mixed", 512), ("mixed", 16), ("wide", 64), ("odd", 5), ("equal", 33)])
def test_portions_of_any_size(env, variant, chunk):
    """A prompt cut into portions (down to two tokens and one) gives the logits of the uncut prompt; `chunk` also cuts long
    portions inside the engine, so attention chunks', key pieces' and tiles' edges fall everywhere and every cut hands over the
    recurrent states and the convolutions' histories (portions shorter than a history included)."""
    cfg = small_config(env["synth"], variant)
    m, _, orc = make(env, cfg, seed=17, TL_STACK_CHUNK=chunk)
    rng = np.random.default_rng(3)
    n = 400 if variant == "wide" else 120
    toks = rng.integers(0, cfg["vocab"], n).astype(np.int32)
    want = orc.forward(list(toks))
    for sizes in ([7, 2, 13, 1, 20, 2, 5, 64, 3], [2] * 20, [1, 1, 1, 2, 1, 3], [n]):
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
    """A second request after reset_kv equals the same request on a fresh model, also when the first one was longer: nothing
    of the first request's keys, recurrent states or convolution histories survives."""
    cfg = small_config(env["synth"], "mixed")
    m, tensors, orc = make(env, cfg, seed=19)
    rng = np.random.default_rng(4)
    a = rng.integers(0, cfg["vocab"], 150).astype(np.int32)
    b = rng.integers(0, cfg["vocab"], 40).astype(np.int32)
    m.prefill_rows(a, 0)
    for i in range(5):
        m.decode(int(a[i]), 150 + i)
    m.reset_kv()
    got = m.prefill_rows(b[:30], 0)
    tail = np.stack([m.decode(int(b[i]), i)[0] for i in range(30, 40)])
    want = orc.forward(list(b))
    assert rel_rms(np.concatenate([got, tail]), want) < FP32_TOL
    m.free()


def test_far_keys_chunk_edges_and_long_states_decide_the_logits(env):
    """Sharpened scores (scale times 6), decays near 1 in every recurrence: logits then rest on a few keys anywhere in the context
    or the chunk and on tokens hundreds of positions back, so that a fault in one of them, or a chunk edge that is one token off,
    moves the logits by far more than the tolerance. Prompt pass, portions, then decoding across chunk edges."""
    synth = env["synth"]
    K, C, D, L = synth.ratuzen_chunked, synth.ratuzen_causal, synth.ratuzen_delta, synth.ratuzen_layer
    cfg = synth.ratuzen_config(64, 97, [
        L("parallel_2", C(4, 2, 16, 16, 2, 16, 16, tau=64.0, factor=2.0, scale=6.0 / math.sqrt(16)), 32),
        L("parallel", K(4, 1, 32, 16, 37, 2, 16, 16, [0.999, 0.995], scale=6.0 / math.sqrt(32)), 32),
        L("delta", D(2, 1, 16, 16), 32),
        L("parallel", K(2, 2, 24, 8, 64, 2, 24, 8, [1.0, 0.9], scale=6.0 / math.sqrt(24)), None)])
    tensors = synth.build_ratuzen(cfg, 23)
    tensors["l2.mix.A_log"] = synth.to_bf16(np.full(2, -6.0, np.float32))
    m, _, orc = make(env, cfg, tensors=tensors)
    rng = np.random.default_rng(5)
    toks = rng.integers(0, cfg["vocab"], 330).astype(np.int32)
    want = orc.forward(list(toks))
    got = [m.prefill_rows(toks[:200], 0), m.prefill_rows(toks[200:230], 200), m.prefill_rows(toks[230:232], 230)]
    got += [m.decode(int(toks[i]), i)[0][None] for i in range(232, 330)]
    assert rel_rms(np.concatenate(got), want) < 2 * FP32_TOL
    # the oracle with a changed chunk, rotation, decay or tau differs by orders of magnitude more: the test can see it
    for path, value in ((("mixer", "left", "mask", "size"), 36), (("mixer", "right", "decay"), [0.998, 0.995])):
        off = json.loads(json.dumps(cfg))
        at = off["layers"][1]
        for key in path[:-1]:
            at = at[key]
        at[path[-1]] = value
        assert rel_rms(env["oracle"].RatuzenOracle(off, tensors).forward(list(toks[:120])), want[:120]) > 40 * FP32_TOL, path
    m.free()


def test_first_tokens_of_a_sequence(env):
    """Positions 0 .. 4, each as a prompt of its own length, as single tokens, and after a reset: the zeros before the start of
    a sequence in every convolution, the empty recurrent states and a one-key softmax."""
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
    """Greedy generation on the device (graph replays back to back) equals the oracle's token-by-token arg-max, well past several
    chunks; the sampled loop is reproducible by seed and stays inside the vocabulary."""
    cfg = small_config(env["synth"], "mixed")
    m, _, orc = make(env, cfg, seed=29)
    prompt = np.array([3, 14, 15, 92, 65, 35], np.int32)
    want = orc.generate_greedy(list(prompt), 120)
    last = m.prefill_rows(prompt, 0, np.array([len(prompt) - 1], np.int32))[0]
    first = int(np.argmax(last))
    more = m.generate_greedy(first, len(prompt), 119)
    assert [first] + list(more) == want
    runs = []
    for _ in range(2):
        m.reset_kv()
        m.prefill_rows(prompt, 0, np.array([len(prompt) - 1], np.int32))
        runs.append(list(m.generate_sampled(first, len(prompt), 30, temperature=0.9, top_k=20, top_p=0.95, seed=7)))
    assert runs[0] == runs[1] and all(0 <= t < cfg["vocab"] for t in runs[0])
    m.free()


def test_graph_replays_match_the_eager_step(env):
    """The captured decode step, replayed many times with prompt work and synchronisations in between, gives the logits of
    the step enqueued launch by launch."""
    cfg = small_config(env["synth"], "mixed")
    rng = np.random.default_rng(8)
    toks = rng.integers(0, cfg["vocab"], 60).astype(np.int32)
    tensors = env["synth"].build_ratuzen(cfg, 37)
    eager, _, _ = make(env, cfg, tensors=tensors, TL_NO_GRAPH=1)
    graph, _, _ = make(env, cfg, tensors=tensors)
    assert graph.graph_captured() and not eager.graph_captured()
    for m in (eager, graph):
        m.prefill_rows(toks[:20], 0, np.array([19], np.int32))
    for i in range(20, 60):
        a, b = eager.decode(int(toks[i]), i)[0], graph.decode(int(toks[i]), i)[0]
        assert np.array_equal(a, b), i
    eager.free()
    graph.free()


@pytest.mark.parametrize("variant", ["mixed", "odd", "wide"])
def test_one_token_step_with_and_without_its_fusions(env, variant):
    """The one-token step as it is served (a recurrence in one launch, the feed-forward on a second stream) against the same step
    with one launch per operation on one stream, against the chunk path fed one token at a time, and against the oracle."""
    cfg = small_config(env["synth"], variant)
    rng = np.random.default_rng(9)
    toks = rng.integers(0, cfg["vocab"], 70).astype(np.int32)
    tensors = env["synth"].build_ratuzen(cfg, 43)
    served, _, orc = make(env, cfg, tensors=tensors)
    plain, _, _ = make(env, cfg, tensors=tensors, TL_STACK_FUSE_STEPS=0, TL_STACK_FORK=0)
    chunked, _, _ = make(env, cfg, tensors=tensors, TL_STACK_GEMV=0)
    assert served.graph_nodes() < plain.graph_nodes()
    want = orc.forward(list(toks))
    outs = []
    for m in (served, plain, chunked):
        m.prefill_rows(toks[:25], 0, np.array([24], np.int32))
        outs.append(np.stack([m.decode(int(toks[i]), i)[0] for i in range(25, 70)]))
        assert rel_rms(outs[-1], want[25:]) < FP32_TOL
        m.free()


def test_generation_through_the_host_session(env, tmp_path):
    """The framework's own entry point: a checkpoint folder opened by tlhost::Session (model registry, config.json reader,
    safetensors loader), greedy generate() for a short and a long prompt, generate_batch over unequal prompts against each
    alone, and the step function a scheduler drives."""
    from tinyllama_cpp_amd import hostapi
    synth = env["synth"]
    cfg = small_config(synth, "mixed")
    tensors = synth.build_ratuzen(cfg, 31)
    synth.write_stack_dir(str(tmp_path / "ckpt"), cfg, tensors)
    orc = env["oracle"].RatuzenOracle(cfg, tensors)
    s = hostapi.Session(str(tmp_path / "ckpt"), 0, 256)
    info = s.info()
    assert info["architecture"] == "Ratuzen" and info["vocab"] == cfg["vocab"] and info["max_pos"] == 256
    s.set_repetition_penalty(1.0)
    s.set_exact(True)
    rng = np.random.default_rng(6)
    for n in (5, 45):
        prompt = rng.integers(0, cfg["vocab"], n).astype(np.int32)
        assert list(s.generate(prompt, steps=24, temperature=0.0)) == orc.generate_greedy(list(prompt), 24)
    prompts = [rng.integers(0, cfg["vocab"], n).astype(np.int32) for n in (3, 40, 11)]
    s.set_max_batch(3)
    outs = s.generate_batch(prompts, steps=10, temperature=0.0)
    for p, o in zip(prompts, outs):
        assert list(o) == orc.generate_greedy(list(p), 10)
    toks = rng.integers(0, cfg["vocab"], 60).astype(np.int32)
    orc.reset()
    want = orc.forward(list(toks))
    s.reset()
    got = [s.forward(toks[:37], 0, [0, 5, 36]), s.forward(toks[37:39], 37, [1])]
    got += [s.forward(toks[i:i + 1], i, [0]) for i in range(39, 60)]
    rows = [0, 5, 36, 38] + list(range(39, 60))
    assert rel_rms(np.concatenate(got), want[rows]) < FP32_TOL
    s.close()


def test_schedule_replayed_by_the_trace_program(env, tmp_path):
    """The command-line program that replays a recorded schedule over a checkpoint folder: a whole prompt, then a second
    request in portions and single tokens after the first one gave its cache and states back; both number formats."""
    import subprocess
    synth = env["synth"]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    exe = os.path.join(root, "tinyllama.cpp_amd", "host", "tl_trace")
    assert os.path.exists(exe), "build the host layer first (make -C tinyllama.cpp_amd/host)"
    cfg = small_config(synth, "mixed")
    tensors = synth.build_ratuzen(cfg, 53)
    synth.write_stack_dir(str(tmp_path / "ckpt"), cfg, tensors)
    orc = env["oracle"].RatuzenOracle(cfg, tensors)
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
    for dtype, tol in (("float32", FP32_TOL), ("bfloat16", BF16_TOL)):
        out = tmp_path / dtype
        out.mkdir()
        r = subprocess.run([exe, "--model", str(tmp_path / "ckpt"), "--dtype", dtype, "--out", str(out), "--max-tokens", "96"],
                           input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
        assert r.returncode == 0, r.stderr
        assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(len(steps))]
        assert not (out / "1.f32").exists()
        got_a = np.fromfile(out / "0.f32", np.float32).reshape(4, cfg["vocab"])
        got_b = np.concatenate([np.fromfile(out / f"{i}.f32", np.float32).reshape(-1, cfg["vocab"]) for i in range(2, len(steps))])
        assert rel_rms(got_a[1:], want_a[1:]) < tol and rel_rms(got_b, want_b) < tol, dtype


def random_config(synth, seed):
    """A configuration drawn at random: layer order, head counts and group ratios, head sizes (also indivisible by 4 and above
    128), chunks, rotations and their scalings, decays, taps, with and without feed-forward."""
    rng = np.random.default_rng(5000 + seed)
    K, C, D, L = synth.ratuzen_chunked, synth.ratuzen_causal, synth.ratuzen_delta, synth.ratuzen_layer
    pick = lambda xs: xs[int(rng.integers(0, len(xs)))]
    layers = []
    for i in range(int(rng.integers(2, 6))):
        kind = pick(["parallel", "parallel_2", "delta"])
        ff, limit = pick([None, 7, 16, 40, 100]), float(pick([0.5, 1.5, 7.0]))
        G = int(pick([1, 2, 3]))
        H, d, dv = G * int(pick([1, 2, 4])), int(pick([6, 10, 16, 32, 64, 136])), int(pick([3, 8, 16, 40, 72]))
        rd = 2 * int(rng.integers(1, d // 2 + 1))
        scale = float(pick([0.1, d ** -0.5, 0.5]))
        base = float(pick([100.0, 10000.0, 500000.0]))
        H2 = int(pick([1, 2, 3]))
        if kind == "parallel":
            sc = pick([None, (4.0, 1.0, 4.0, 64), (8.0, 1.0, 4.0, 512), (1.5, 0.5, 3.0, 30)])
            layers.append(L(kind, K(H, G, d, dv, int(pick([0, 1, 2, 7, 33, 64, 100])), H2, int(pick([3, 8, 16, 64, 130])), int(pick([3, 8, 20, 64])),
                                    [float(pick([0.0, 0.3, 0.9, 0.999, 1.0])) for _ in range(H2)], base=base, rot_dims=rd, scaling=sc, scale=scale), ff, limit))
        elif kind == "parallel_2":
            layers.append(L(kind, C(H, G, d, dv, H2, int(pick([3, 8, 16, 24, 64, 130])), int(pick([3, 8, 20, 64])), tau=float(pick([1.0, 4.0, 16.0])),
                                    base=base, rot_dims=rd, factor=pick([None, 1.0, 4.0]), scale=scale), ff, limit))
        else:
            layers.append(L(kind, D(H, G, int(pick([3, 8, 16, 64, 130])), int(pick([3, 8, 20])), conv=int(pick([1, 2, 4]))), ff, limit))
    return synth.ratuzen_config(int(pick([24, 50, 64, 100])), int(pick([40, 97, 130])), layers, eps=float(pick([1e-6, 1e-5, 1e-2])),
                                logit_scale=float(pick([0.1, 1.0, 3.0]))), int(pick([1, 4, 8, 17]))


@pytest.mark.parametrize("seed", range(16))
def test_configurations_drawn_at_random(env, seed, tmp_path):
    """Through the host session over a checkpoint folder (so the configuration reader is part of what is tested): a prompt in
    portions and decoded tokens against the oracle, twice over so that state and cache are given back in between."""
    from tinyllama_cpp_amd import hostapi
    synth = env["synth"]
    cfg, rank = random_config(synth, seed)
    tensors = synth.build_ratuzen(cfg, seed, rank=rank)
    synth.write_stack_dir(str(tmp_path / "ckpt"), cfg, tensors)
    orc = env["oracle"].RatuzenOracle(cfg, tensors)
    rng = np.random.default_rng(seed)
    n = 150
    s = hostapi.Session(str(tmp_path / "ckpt"), 0, n)
    s.set_exact(True)
    for _ in range(2):
        toks = rng.integers(0, cfg["vocab"], n).astype(np.int32)
        orc.reset()
        want = orc.forward(list(toks))
        s.reset()
        got, p = [], 0
        for size in [int(x) for x in rng.integers(1, 24, 6)] + [2]:
            got.append(s.forward(toks[p:p + size], p, list(range(size))))
            p += size
        got += [s.forward(toks[i:i + 1], i, [0]) for i in range(p, n)]
        # (four times the usual bound: drawn sizes include head norms over three channels, which magnify the last bits of single
        #  rows)
        assert rel_rms(np.concatenate(got), want) < 4 * FP32_TOL, json.dumps(cfg)
    s.close()
