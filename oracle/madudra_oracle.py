"""Plain, slow float64 implementation of the Madudra layer-list design: test infrastructure only.

One function per mechanism, written from the equations, sharing nothing with the product path (libtlhip.so); numpy only.
Weights arrive as {checkpoint name: uint16 array of bf16 bits}; `config` is config.json's dictionary.

  embedding   e = embed[token] * embedding.scale; each of the `streams` residual streams starts as e
  sublayer    with a_in [S], a_out [S], M [S, S] of the sublayer: u = sum_s a_in[s] x_s;  y = f(norm(u));
              x_t <- sum_s M[s, t] x_s + residual_mult a_out[t] y, every stream from the old ones
  norm        (x - mean) / sqrt(var + eps) * w, var the mean squared deviation, no bias
  latent attention   c_q = rms(W_dq h) w_q; q = W_uq c_q, per head [plain | rotated]; [c | r] = W_dkv h, c <- rms(c) w_kv; the
              rotated parts turn by position (halves paired: i with i + dims / 2; blended frequencies); head n's key
              [W_uk,n c | r], value W_uv,n c; softmax of (q . k) scale over 0 <= i - j < window; heads times sigmoid(W_g h); W_o.
              kv_from: c and r come from an earlier layer's cache
  mamba2      [z | x | B | C | dt] = W_in h; (x, B, C) through a causal convolution per channel + bias + silu;
              dt <- softplus(dt + dt_bias); per head S <- exp(-exp(A_log) dt) S + dt B x^T, y = S^T C + D x (B, C shared by the
              heads of a group); y silu(z), RMS norm in equal parts, weight; W_o
  experts     s = softmax(W_router h); the `top` largest; weights = their s times router.scale;
              expert: W_down gelu(W_up h), gelu(z) = z Phi(z)
  output      sum of the streams, norm, head
"""
import math

import numpy as np


def widen(bits):
    return (np.asarray(bits, np.uint16).astype(np.uint32) << 16).view(np.float32).astype(np.float64)


def sigmoid(z):
    return np.exp(-np.logaddexp(0.0, -z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


_erf = np.vectorize(math.erf, otypes=[np.float64])


def gelu(z):
    return 0.5 * z * (1.0 + _erf(z / math.sqrt(2.0)))


def rms(x, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def layer_norm(x, w, eps):
    d = x - x.mean(-1, keepdims=True)
    return d / np.sqrt((d * d).mean(-1, keepdims=True) + eps) * w


def streams_in(xs, a_in):
    """xs [T, S, W] -> sum_s a_in[s] x_s."""
    return sum(a_in[s] * xs[:, s] for s in range(xs.shape[1]))


def streams_out(xs, y, mix, a_out, m):
    """The streams after a sublayer whose output is y [T, W]; mix is indexed [from, to]."""
    S = xs.shape[1]
    return np.stack([sum(mix[s, t] * xs[:, s] for s in range(S)) + m * a_out[t] * y for t in range(S)], axis=1)


def rotary_frequencies(dims, base, scaling=None):
    """(f [dims / 2], factor on cos and sin)."""
    i = np.arange(dims // 2, dtype=np.float64)
    f = float(base) ** (-2.0 * i / dims)
    if not scaling:
        return f, 1.0
    at = lambda turns: dims * math.log(scaling["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(at(scaling["fast"])), 0)
    hi = min(math.ceil(at(scaling["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / scaling["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(scaling["factor"]) + 1.0


def rotate_halves(x, pos, dims, f, mscale):
    """x [T, ..., d] at positions pos: dimension i turns with i + dims / 2, the dimensions from `dims` on pass."""
    out = x.copy()
    half = dims // 2
    for t in range(x.shape[0]):
        c, s = np.cos(pos[t] * f) * mscale, np.sin(pos[t] * f) * mscale
        u, v = x[t, ..., :half], x[t, ..., half:dims]
        out[t, ..., :half] = u * c - v * s
        out[t, ..., half:dims] = v * c + u * s
    return out


def softmax_attention(q, k, v, scale, q_pos, window=0):
    """q [T, H, d] at positions q_pos, k [P, H, d], v [P, H, vd] (key j at position j) -> [T, H, vd]."""
    T, H, _ = q.shape
    out = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        i = int(q_pos[t])
        lo = max(0, i - window + 1) if window > 0 else 0
        for h in range(H):
            s = (k[lo:i + 1, h] @ q[t, h]) * scale
            e = np.exp(s - s.max())
            out[t, h] = (e @ v[lo:i + 1, h]) / e.sum()
    return out


def causal_conv(u, w, bias, hist):
    """u [T, C] inputs, w [C, taps] (the last column is the current token's), hist [taps - 1, C] the inputs before u (oldest
    first) -> (y [T, C], the new history)."""
    taps = w.shape[1]
    full = np.concatenate([hist, u]) if taps > 1 else u
    y = np.zeros_like(u) + bias
    for j in range(taps):
        y = y + full[j:j + u.shape[0]] * w[:, j]
    return y, (full[full.shape[0] - (taps - 1):] if taps > 1 else hist)


def state_space(x, B, C, dt, rate, D, S):
    """One head: x [T, vd], B, C [T, N], dt [T], S [N, vd] updated in place: S <- exp(-rate dt) S + dt B x^T; y = S^T C + D x."""
    y = np.zeros_like(x)
    for t in range(x.shape[0]):
        S[:] = math.exp(-rate * dt[t]) * S + dt[t] * np.outer(B[t], x[t])
        y[t] = S.T @ C[t] + D * x[t]
    return y


def gated_part_norm(y, z, parts, eps, w):
    """y silu(z), then an RMS norm in `parts` equal parts of the row, then the weight."""
    g = (y * silu(z)).reshape(y.shape[0], parts, -1)
    return rms(g, eps).reshape(y.shape) * w


def route_softmax(z, top, scale):
    """z [E] router logits -> (ids [top] largest first, weights: the softmax over ALL experts, scaled, not renormalised)."""
    e = np.exp(z - z.max())
    s = e / e.sum()
    ids = np.argsort(-s, kind="stable")[:top]
    return ids, s[ids] * scale


class MadudraOracle:
    def __init__(self, config, tensors):
        self.c = config
        self.w = {k: widen(v) for k, v in tensors.items()}
        self.eps = config["norm"]["eps"]
        self.reset()

    def reset(self):
        self.state = [dict() for _ in self.c["layers"]]
        self.pos = 0

    def latent_attention(self, i, h, pos):
        mx, p, w = self.c["layers"][i]["mixer"], f"l{i}.mix.", self.w
        T, H, d, rd, vd, rk = h.shape[0], mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
        rot = mx["rot"]
        f, mscale = rotary_frequencies(rot["dims"], rot["base"], rot.get("scaling"))
        cq = rms(h @ w[p + "dq"].T, self.eps) * w[p + "dq.norm"]
        q = (cq @ w[p + "uq"].T).reshape(T, H, d + rd)
        q = np.concatenate([q[..., :d], rotate_halves(q[..., d:], pos, rot["dims"], f, mscale)], axis=-1)
        if mx.get("kv_from") is None:
            kv = h @ w[p + "dkv"].T
            rows = np.concatenate([rms(kv[:, :rk], self.eps) * w[p + "dkv.norm"],
                                   rotate_halves(kv[:, rk:], pos, rot["dims"], f, mscale)], axis=1)
            old = self.state[i].get("rows")
            self.state[i]["rows"] = rows if old is None else np.concatenate([old, rows])
        rows = self.state[i if mx.get("kv_from") is None else mx["kv_from"]]["rows"]
        P = rows.shape[0]
        c, r = rows[:, :rk], rows[:, rk:]
        k = np.concatenate([(c @ w[p + "uk"].T).reshape(P, H, d), np.repeat(r[:, None], H, axis=1)], axis=-1)
        v = (c @ w[p + "uv"].T).reshape(P, H, vd)
        o = softmax_attention(q, k, v, mx["scale"], pos, (mx.get("mask") or {}).get("size", 0)).reshape(T, -1)
        return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T

    def mamba2(self, i, h):
        mx, p, w = self.c["layers"][i]["mixer"], f"l{i}.mix.", self.w
        T, H, vd, N, G = h.shape[0], mx["heads"], mx["vdim"], mx["state"], mx["groups"]
        inner, C = H * vd, H * vd + 2 * G * N
        u = h @ w[p + "in"].T
        z, xbc, dt = u[:, :inner], u[:, inner:inner + C], u[:, inner + C:]
        hist = self.state[i].get("conv")
        if hist is None:
            hist = np.zeros((mx["conv"] - 1, C))
        xbc, self.state[i]["conv"] = causal_conv(xbc, w[p + "conv"], w[p + "conv.b"], hist)
        xbc = silu(xbc)
        x = xbc[:, :inner].reshape(T, H, vd)
        B = xbc[:, inner:inner + G * N].reshape(T, G, N)
        Cm = xbc[:, inner + G * N:].reshape(T, G, N)
        dt = softplus(dt + w[p + "dt_bias"])
        S = self.state[i].setdefault("S", np.zeros((H, N, vd)))
        y = np.stack([state_space(x[:, n], B[:, n // (H // G)], Cm[:, n // (H // G)], dt[:, n], math.exp(w[p + "A_log"][n]),
                                  w[p + "D"][n], S[n]) for n in range(H)], axis=1).reshape(T, inner)
        return gated_part_norm(y, z, mx["norm_groups"], self.eps, w[p + "norm"]) @ w[p + "o"].T

    def experts(self, i, h):
        m, p, w = self.c["layers"][i]["mlp"], f"l{i}.mlp.", self.w
        r = m["router"]
        z = h @ w[p + "router"].T
        out = np.zeros_like(h)
        for t in range(h.shape[0]):
            for e, a in zip(*route_softmax(z[t], r["top"], r["scale"])):
                out[t] += a * (gelu(h[t] @ w[f"{p}e{e}.up"].T) @ w[f"{p}e{e}.down"].T)
        return out

    def sublayer(self, i, q, xs, f):
        p, w = f"l{i}.hc{q}.", self.w
        u = streams_in(xs, w[p + "in"])
        y = f(layer_norm(u, w[f"l{i}.norm{q}"], self.eps))
        return streams_out(xs, y, w[p + "mix"], w[p + "out"], self.c["residual_mult"])

    def forward(self, tokens, residuals=None):
        """The next tokens of the sequence: logits [T, vocab]. residuals: a list that receives the streams' sum after every layer."""
        T = len(tokens)
        pos = np.arange(self.pos, self.pos + T)
        e = self.w["embed"][np.asarray(tokens)] * self.c["embedding"]["scale"]
        xs = np.repeat(e[:, None], self.c["streams"], axis=1)
        for i, L in enumerate(self.c["layers"]):
            if L["type"] == "latent_attention":
                xs = self.sublayer(i, 1, xs, lambda h: self.latent_attention(i, h, pos))
            elif L["type"] == "mamba2":
                xs = self.sublayer(i, 1, xs, lambda h: self.mamba2(i, h))
            else:
                raise ValueError(f"unknown layer type {L['type']!r}")
            if L.get("mlp") is not None:
                xs = self.sublayer(i, 2, xs, lambda h: self.experts(i, h))
            if residuals is not None:
                residuals.append(xs.sum(1))
        self.pos += T
        return layer_norm(xs.sum(1), self.w["final.norm"], self.eps) @ self.w["head"].T

    def generate_greedy(self, prompt, n_new):
        """Arg-max continuation (first maximum), token by token after the prompt; resets the sequence first."""
        self.reset()
        logits = self.forward(list(prompt))[-1]
        out = []
        for _ in range(n_new):
            out.append(int(np.argmax(logits)))
            logits = self.forward([out[-1]])[0]
        return out
