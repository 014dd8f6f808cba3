"""Plain float64 restatement of the Rudilix decoder, one function per mechanism, written token by
token and key by key.  It shares nothing with the HIP path: numpy only, no caches, no chunks, no
fused weights.  ``weights`` is a dict of checkpoint tensors by name; ``config`` the parsed
config.json.

Sequences are processed from an explicit recurrent state so that a test can also feed a prompt
in pieces; ``State`` holds what a layer carries from one token to the next.
"""
from __future__ import annotations

import numpy as np

F = np.float64


def sigmoid(x):
    x = np.asarray(x, F)
    e = np.exp(-np.abs(x))
    return np.where(x >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return np.maximum(x, 0.0) + np.log1p(np.exp(-np.abs(x)))


def rms(x, eps):
    """x over the root of its mean square (last axis), eps under the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rms_norm_plus_one(x, w, eps):
    return rms(x, eps) * (1.0 + w)


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def causal_conv(x, w, b=None, past=None):
    """out[t, c] = b[c] + sum_j w[c, j] * in[t - (taps - 1) + j, c]; inputs before the start are ``past``
    (the taps - 1 inputs before x, oldest first), or zero.  Returns (out, the new past)."""
    taps = w.shape[1]
    T, C = x.shape
    if past is None:
        past = np.zeros((taps - 1, C))
    full = np.concatenate([past, x], 0)
    out = np.zeros((T, C))
    for t in range(T):
        for j in range(taps):
            out[t] += w[:, j] * full[t + j]
    if b is not None:
        out = out + b
    return out, full[len(full) - (taps - 1):]


def rotate(x, pos, dims, base):
    """Interleaved rotary on the first ``dims`` entries of x [..., D] at position ``pos``."""
    x = x.copy()
    for i in range(dims // 2):
        a = pos * base ** (-2.0 * i / dims)
        u, v = x[..., 2 * i].copy(), x[..., 2 * i + 1].copy()
        x[..., 2 * i] = u * np.cos(a) - v * np.sin(a)
        x[..., 2 * i + 1] = v * np.cos(a) + u * np.sin(a)
    return x


def window_attention(q, k, v, first, size, scale):
    """q [T, H, D] at positions first .. first + T; k [P, G, D], v [P, G, E] of positions 0 .. P.
    Position i sees j with 0 <= i - j < size.  Returns [T, H, E]."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        i = first + t
        lo = max(0, i - size + 1)
        for h in range(H):
            g = h // (H // G)
            s = (k[lo:i + 1, g] @ q[t, h]) * scale
            p = np.exp(s - s.max())
            out[t, h] = (p / p.sum()) @ v[lo:i + 1, g]
    return out


def delta_rule(S, q, k, v, g, beta):
    """One head: S [D, E], q/k/g [T, D], v [T, E], beta [T].  Decay the rows, correct towards v, read out."""
    S = S.copy()
    o = np.zeros_like(v)
    for t in range(len(q)):
        S = g[t][:, None] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + np.outer(k[t], u)
        o[t] = S.T @ q[t]
    return o, S


def ssd(S, x, B, C, dt, a_log, D):
    """One head: S [N, P], x [T, P], B/C [T, N], dt [T] (after softplus), scalars a_log and D."""
    S = S.copy()
    y = np.zeros_like(x)
    for t in range(len(x)):
        S = np.exp(-np.exp(a_log) * dt[t]) * S + dt[t] * np.outer(B[t], x[t])
        y[t] = S.T @ C[t] + D * x[t]
    return y, S


def clamped_glu(h, w_gate, w_up, w_down, limit):
    g = np.minimum(h @ w_gate.T, limit)
    u = np.clip(h @ w_up.T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w_down.T


def mamba2_mixer(h, w, c, eps, st):
    H, P, N, G = c["heads"], c["vdim"], c["state"], c["groups"]
    inner = H * P
    proj = h @ w("in").T
    z, xbc, dt = proj[:, :inner], proj[:, inner:2 * inner + 2 * G * N], proj[:, 2 * inner + 2 * G * N:]
    xbc, st["conv"] = causal_conv(xbc, w("conv"), w("conv.b"), st.get("conv"))
    xbc = silu(xbc)
    x = xbc[:, :inner].reshape(-1, H, P)
    B = xbc[:, inner:inner + G * N].reshape(-1, G, N)
    C = xbc[:, inner + G * N:].reshape(-1, G, N)
    dt = softplus(dt + w("dt_bias"))
    S = st.get("S", np.zeros((H, N, P)))
    y, new = np.zeros_like(x), np.zeros_like(S)
    for hd in range(H):
        g = hd // (H // G)
        y[:, hd], new[hd] = ssd(S[hd], x[:, hd], B[:, g], C[:, g], dt[:, hd], w("A_log")[hd], w("D")[hd])
    st["S"] = new
    y = y.reshape(-1, inner) * silu(z)
    y = rms(y.reshape(len(y), c["norm_groups"], -1), eps).reshape(-1, inner) * w("norm")
    return y @ w("o").T


def delta_mixer(h, w, c, eps, st):
    H, G, D, E = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    qkv = []
    for n in "qkv":
        p, st["conv." + n] = causal_conv(h @ w(n).T, w(n + ".conv"), None, st.get("conv." + n))
        qkv.append(silu(p))
    q = unit(qkv[0].reshape(-1, G, D)) * D ** -0.5
    k = unit(qkv[1].reshape(-1, G, D))
    v = qkv[2].reshape(-1, H, E)
    beta = sigmoid(h @ w("b").T)
    raw = ((h @ w("a1").T) @ w("a2").T + w("dt_bias")).reshape(-1, H, D)
    g = np.exp(-np.exp(w("A_log"))[:, None] * softplus(raw))
    S = st.get("S", np.zeros((H, D, E)))
    o, new = np.zeros_like(v), np.zeros_like(S)
    for hd in range(H):
        j = hd // (H // G)
        o[:, hd], new[hd] = delta_rule(S[hd], q[:, j], k[:, j], v[:, hd], g[:, hd], beta[:, hd])
    st["S"] = new
    gate = sigmoid((h @ w("g1").T) @ w("g2").T).reshape(-1, H, E)
    o = rms(o, eps) * w("norm") * gate
    return o.reshape(len(h), -1) @ w("o").T


def attention_mixer(h, w, c, eps, st, first):
    H, G, D, E = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q = (h @ w("q").T + w("q.b")).reshape(-1, H, D)
    k = (h @ w("k").T + w("k.b")).reshape(-1, G, D)
    v = (h @ w("v").T + w("v.b")).reshape(-1, G, E)
    q, k = rms(q, eps) * w("q.norm"), rms(k, eps) * w("k.norm")
    for t in range(len(h)):
        q[t] = rotate(q[t], first + t, c["rot"]["dims"], c["rot"]["base"])
        k[t] = rotate(k[t], first + t, c["rot"]["dims"], c["rot"]["base"])
    k = np.concatenate([st["k"], k], 0) if "k" in st else k
    v = np.concatenate([st["v"], v], 0) if "v" in st else v
    st["k"], st["v"] = k, v
    o = window_attention(q, k, v, first, c["mask"]["size"], c["scale"])
    o = o * sigmoid(h @ w("g").T)[:, :, None]
    return o.reshape(len(h), -1) @ w("o").T


def mixer(kind, h, w, c, eps, st, first):
    if kind == "mamba2":
        return mamba2_mixer(h, w, c, eps, st)
    if kind == "channel_delta":
        return delta_mixer(h, w, c, eps, st)
    if kind == "parallel":
        left = attention_mixer(h, lambda n: w("left." + n), c["left"], eps, st.setdefault("left", {}), first)
        right = delta_mixer(h, lambda n: w("right." + n), c["right"], eps, st.setdefault("right", {}))
        return c["left_scale"] * left + c["right_scale"] * right
    raise ValueError(kind)


class Sequence:
    """A sequence in progress: ``run(tokens)`` returns the logits of these tokens (and, if a list is
    given, appends the residual stream after every layer)."""

    def __init__(self, config, weights):
        self.c = config
        self.w = {n: np.asarray(t, F) for n, t in weights.items()}
        self.first = 0
        self.states = [{} for _ in config["layers"]]

    def run(self, tokens, layers=None):
        c, eps, m = self.c, self.c["norm"]["eps"], self.c["residual_mult"]
        x = self.w["embed"][np.asarray(tokens, np.int64)]
        for i, layer in enumerate(c["layers"]):
            p = f"l{i}."
            h = rms_norm_plus_one(x, self.w[p + "norm1"], eps)
            x = x + m * mixer(layer["type"], h, lambda n: self.w[p + "mix." + n], layer["mixer"], eps, self.states[i], self.first)
            if layer["mlp"] is not None:
                h = rms_norm_plus_one(x, self.w[p + "norm2"], eps)
                x = x + m * clamped_glu(h, self.w[p + "mlp.gate"], self.w[p + "mlp.up"], self.w[p + "mlp.down"],
                                        layer["mlp"]["limit"])
            if layers is not None:
                layers.append(x)
        self.first += len(tokens)
        return rms_norm_plus_one(x, self.w["final.norm"], eps) @ self.w["head"].T
