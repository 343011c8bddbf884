"""Plain, slow float64 implementation of the Ratuzen layer-list design: test infrastructure only.

One function per mechanism, written from the equations, sharing nothing with the product path (libtlhip.so); numpy only.
Weights arrive as {checkpoint name: uint16 array of bf16 bits}; `config` is config.json's dictionary.

  norm        N(x; w) = x / sqrt(mean(x^2) + eps) * w
  layer       x <- x + mixer(N(x; norm1)) + ff(N(x; norm2)): both sublayers read the same x
  mixers      parallel    1/2 (N(left(h); left.out) + N(right(h); right.out)), left = rotated attention inside chunks with biases on
                          q, k, v and wavelength-dependent frequency scaling, right = linear attention with one constant decay
                          per head on silu-activated q, k, v, one norm over all heads, a sigmoid gate per column
              parallel_2  the same combination, left = causal attention with q/k RMS norms per head in front of a half-paired
                          rotation at frequencies divided by a factor and a sigmoid gate per head, right = linear attention with a
                          decay per key channel sigmoid(z)^(1/tau), a norm per head, a silu gate per column
              delta       gated delta rule with one decay per head behind short convolutions
  ff          g = min(W_gate h, L), u = clip(W_up h, -L, L); W_down (g sigmoid(1.702 g) (u + 1))
  output      logit_scale * head N(x; final.norm)
"""
import math

import numpy as np


def widen(bits):
    return (np.asarray(bits, np.uint16).astype(np.uint32) << 16).view(np.float32).astype(np.float64)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def rms(x, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def frequencies(rot):
    """The rot['dims'] / 2 angular frequencies, scaled as rot['scaling'] says: a factor alone divides all of them; with low,
    high, original the slow ones are divided, the fast ones stay and those between are blended by wavelength."""
    n = rot["dims"]
    f = np.array([rot["base"] ** (-2.0 * i / n) for i in range(n // 2)])
    sc = rot.get("scaling")
    if not sc:
        return f
    if "original" not in sc:
        return f / sc["factor"]
    out = []
    for fi in f:
        wavelength = 2.0 * math.pi / fi
        if wavelength < sc["original"] / sc["high"]:
            out.append(fi)
        elif wavelength > sc["original"] / sc["low"]:
            out.append(fi / sc["factor"])
        else:
            s = (sc["original"] / wavelength - sc["low"]) / (sc["high"] - sc["low"])
            out.append((1.0 - s) * fi / sc["factor"] + s * fi)
    return np.array(out)


def rotate(x, pos, freq, halves):
    """x [T, H, d] at positions pos: the first 2 len(freq) dimensions turn in pairs (2i, 2i + 1), or (i, i + len(freq)) with halves."""
    y = x.copy()
    n = len(freq)
    a = np.asarray(pos, np.float64)[:, None] * freq[None, :]
    c, s = np.cos(a)[:, None, :], np.sin(a)[:, None, :]
    first = np.arange(n) if halves else 2 * np.arange(n)
    second = first + n if halves else first + 1
    u, v = x[..., first], x[..., second]
    y[..., first] = u * c - v * s
    y[..., second] = v * c + u * s
    return y


def first_visible(i, chunk):
    """The first key position that position i sees (chunk 0: all of them)."""
    return i // chunk * chunk if chunk > 0 else 0


def softmax_attention(q, k, v, scale, q_pos, chunk=0):
    """q [T, H, d] at positions q_pos, k [P, G, d], v [P, G, vd] (key j at position j) -> [T, H, vd]; chunk > 0: position i sees
    j <= i only where floor(i / chunk) = floor(j / chunk)."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        i = int(q_pos[t])
        lo = first_visible(i, chunk)
        for h in range(H):
            g = h // (H // G)
            s = (k[lo:i + 1, g] @ q[t, h]) * scale
            e = np.exp(s - s.max())
            out[t, h] = (e @ v[lo:i + 1, g]) / e.sum()
    return out


def linear_recurrence(q, k, v, decay, S):
    """One head: q, k [T, d], v [T, vd], decay [T, d] (or broadcastable to it), S [d, vd] updated in place:
    S <- diag(decay) S + k v^T; o = S^T q."""
    decay = np.broadcast_to(decay, k.shape)
    o = np.zeros((q.shape[0], S.shape[1]))
    for t in range(q.shape[0]):
        S[:] = decay[t][:, None] * S + np.outer(k[t], v[t])
        o[t] = S.T @ q[t]
    return o


def gated_delta_rule(q, k, v, beta, g, S):
    """One head: q, k [T, d], v [T, vd], beta, g [T], S [d, vd] updated in place."""
    o = np.zeros((q.shape[0], S.shape[1]))
    for t in range(q.shape[0]):
        S *= g[t]
        u = beta[t] * (v[t] - S.T @ k[t])
        S += np.outer(k[t], u)
        o[t] = S.T @ q[t]
    return o


def causal_conv(u, w, hist):
    """u [T, C] inputs, w [C, taps] (the last column is the current token's), hist [taps - 1, C] the inputs before u (oldest
    first) -> (y [T, C], the new history)."""
    taps = w.shape[1]
    full = np.concatenate([hist, u]) if taps > 1 else u
    y = np.zeros_like(u)
    for j in range(taps):
        y += full[j:j + u.shape[0]] * w[:, j]
    return y, (full[full.shape[0] - (taps - 1):] if taps > 1 else hist)


def clamped_unit(h, gate, up, down, limit):
    g = np.minimum(h @ gate.T, limit)
    u = np.clip(h @ up.T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ down.T


class RatuzenOracle:
    def __init__(self, config, tensors):
        self.c = config
        self.w = {k: widen(v) for k, v in tensors.items()}
        self.eps = config["norm"]["eps"]
        self.reset()

    def reset(self):
        self.state = [dict() for _ in self.c["layers"]]
        self.pos = 0

    def norm(self, name, x):
        return rms(x, self.eps) * self.w[name]

    def append(self, i, key, rows):
        old = self.state[i].get(key)
        self.state[i][key] = rows if old is None else np.concatenate([old, rows])
        return self.state[i][key]

    def conv(self, i, name, u):
        w = self.w[name + ".conv"]
        hist = self.state[i].get(name)
        if hist is None:
            hist = np.zeros((w.shape[1] - 1, u.shape[1]))
        y, self.state[i][name] = causal_conv(u, w, hist)
        return silu(y)

    def chunk_attention(self, i, mx, p, h, pos):
        w = self.w
        T, H, G, d, vd = h.shape[0], mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
        q, k, v = (h @ w[p + n].T + w[p + n + ".b"] for n in "qkv")
        f = frequencies(mx["rot"])
        q = rotate(q.reshape(T, H, d), pos, f, False)
        k = self.append(i, "k", rotate(k.reshape(T, G, d), pos, f, False))
        v = self.append(i, "v", v.reshape(T, G, vd))
        o = softmax_attention(q, k, v, mx["scale"], pos, (mx.get("mask") or {}).get("size", 0))
        return o.reshape(T, -1) @ w[p + "o"].T

    def normed_attention(self, i, mx, p, h, pos):
        w = self.w
        T, H, G, d, vd = h.shape[0], mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
        f = frequencies(mx["rot"])
        q = rms((h @ w[p + "q"].T).reshape(T, H, d), self.eps) * w[p + "q.norm"]
        k = rms((h @ w[p + "k"].T).reshape(T, G, d), self.eps) * w[p + "k.norm"]
        q = rotate(q, pos, f, True)
        k = self.append(i, "k", rotate(k, pos, f, True))
        v = self.append(i, "v", (h @ w[p + "v"].T).reshape(T, G, vd))
        o = softmax_attention(q, k, v, mx["scale"], pos)
        o = o * sigmoid(h @ w[p + "g"].T)[:, :, None]
        return o.reshape(T, -1) @ w[p + "o"].T

    def constant_decay_attention(self, i, mx, p, h):
        w = self.w
        T, H, d, vd = h.shape[0], mx["heads"], mx["dim"], mx["vdim"]
        q, k = (silu(h @ w[p + n].T).reshape(T, H, d) for n in "qk")
        v = silu(h @ w[p + "v"].T).reshape(T, H, vd)
        S = self.state[i].setdefault("S", np.zeros((H, d, vd)))
        o = np.stack([linear_recurrence(q[:, n], k[:, n], v[:, n], mx["decay"][n], S[n]) for n in range(H)], axis=1)
        o = rms(o.reshape(T, -1), self.eps) * w[p + "norm"]
        return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T

    def channel_decay_attention(self, i, mx, p, h):
        w = self.w
        T, H, d, vd = h.shape[0], mx["heads"], mx["dim"], mx["vdim"]
        q = (h @ w[p + "q"].T).reshape(T, H, d) * d ** -0.5
        k = (h @ w[p + "k"].T).reshape(T, H, d)
        v = (h @ w[p + "v"].T).reshape(T, H, vd)
        z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
        alpha = np.exp(-softplus(-z) / mx["tau"]).reshape(T, H, d)
        S = self.state[i].setdefault("S", np.zeros((H, d, vd)))
        o = np.stack([linear_recurrence(q[:, n], k[:, n], v[:, n], alpha[:, n], S[n]) for n in range(H)], axis=1)
        o = (rms(o, self.eps) * w[p + "norm"]).reshape(T, -1)
        return (o * silu(h @ w[p + "g"].T)) @ w[p + "o"].T

    def delta_rule(self, i, mx, p, h):
        w = self.w
        T, H, G, d, vd = h.shape[0], mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
        q, k, v = (self.conv(i, p + n, h @ w[p + n].T) for n in "qkv")
        q = q.reshape(T, G, d)
        k = k.reshape(T, G, d)
        q = q / np.sqrt((q * q).sum(-1, keepdims=True) + 1e-6) * d ** -0.5
        k = k / np.sqrt((k * k).sum(-1, keepdims=True) + 1e-6)
        v = v.reshape(T, H, vd)
        beta = sigmoid(h @ w[p + "b"].T)
        g = np.exp(-np.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
        S = self.state[i].setdefault("S", np.zeros((H, d, vd)))
        o = np.stack([gated_delta_rule(q[:, n // (H // G)], k[:, n // (H // G)], v[:, n], beta[:, n], g[:, n], S[n])
                      for n in range(H)], axis=1)
        o = (rms(o, self.eps) * w[p + "norm"]).reshape(T, -1) * silu(h @ w[p + "g"].T)
        return o @ w[p + "o"].T

    def mixer(self, i, h, pos):
        L, p = self.c["layers"][i], f"l{i}.mix."
        mx = L["mixer"]
        if L["type"] == "delta":
            return self.delta_rule(i, mx, p, h)
        if L["type"] == "parallel":
            left = self.chunk_attention(i, mx["left"], p + "left.", h, pos)
            right = self.constant_decay_attention(i, mx["right"], p + "right.", h)
        elif L["type"] == "parallel_2":
            left = self.normed_attention(i, mx["left"], p + "left.", h, pos)
            right = self.channel_decay_attention(i, mx["right"], p + "right.", h)
        else:
            raise ValueError(f"unknown layer type {L['type']!r}")
        return 0.5 * (self.norm(p + "left.out", left) + self.norm(p + "right.out", right))

    def ff(self, i, h):
        m, p, w = self.c["layers"][i]["mlp"], f"l{i}.mlp.", self.w
        if m["kind"] != "dense":
            raise ValueError("unknown feed-forward kind")
        return clamped_unit(h, w[p + "gate"], w[p + "up"], w[p + "down"], m["limit"])

    def forward(self, tokens, residuals=None):
        """The next tokens of the sequence: logits [T, vocab]. residuals: a list that receives x after every layer."""
        T = len(tokens)
        pos = np.arange(self.pos, self.pos + T)
        x = self.w["embed"][np.asarray(tokens)]
        for i, L in enumerate(self.c["layers"]):
            y = self.mixer(i, self.norm(f"l{i}.norm1", x), pos)
            if L.get("mlp") is not None:
                y = y + self.ff(i, self.norm(f"l{i}.norm2", x))
            x = x + y
            if residuals is not None:
                residuals.append(x.copy())
        self.pos += T
        return (self.norm("final.norm", x) @ self.w["head"].T) * self.c["logit_scale"]

    def generate_greedy(self, prompt, n_new):
        """Arg-max continuation (first maximum), token by token after the prompt; resets the sequence first."""
        self.reset()
        logits = self.forward(list(prompt))[-1]
        out = []
        for _ in range(n_new):
            out.append(int(np.argmax(logits)))
            logits = self.forward([out[-1]])[0]
        return out
