"""Plain float64 restatement of the Lomozen decoder, one function per mechanism, written token by token and key by
key.  It shares nothing with the HIP path: numpy only, no pages, no chunks, no fused weights.  ``weights`` is a dict of
checkpoint tensors by name; ``config`` the parsed config.json.

A ``Sequence`` holds what every layer carries from one token to the next, so that a test can feed a prompt in pieces.
"""
from __future__ import annotations

import math

import numpy as np

F = np.float64


def sigmoid(x):
    x = np.asarray(x, F)
    e = np.exp(-np.abs(x))
    return np.where(x >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(x):
    return x * sigmoid(x)


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def yarn(dims, base, scaling):
    """(frequencies [dims / 2], factor of cosine and sine)."""
    freq = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return np.array(freq), 1.0
    factor, original = scaling["factor"], scaling["original"]

    def turns(t):  # the dimension that turns t times within the original length
        return dims * math.log(original / (2.0 * math.pi * t)) / (2.0 * math.log(base))
    lo = max(math.floor(turns(scaling["fast"])), 0)
    hi = min(math.ceil(turns(scaling["slow"])), dims - 1)
    out = []
    for i, f in enumerate(freq):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / factor * ramp + f * (1.0 - ramp))
    return np.array(out), 0.1 * math.log(factor) + 1.0


def rotate_half(x, pos, dims, base, scaling=None):
    """Entries i and i + dims / 2 of the last axis are a pair; entries past ``dims`` stay."""
    freq, m = yarn(dims, base, scaling)
    x = np.array(x, F)
    for i in range(dims // 2):
        a = pos * freq[i]
        c, s = m * math.cos(a), m * math.sin(a)
        u, v = x[..., i].copy(), x[..., i + dims // 2].copy()
        x[..., i] = u * c - v * s
        x[..., i + dims // 2] = v * c + u * s
    return x


def window_attention(q, k, v, first, size, scale):
    """q [T, H, D] at positions first .. first + T; k [P, H, D], v [P, H, E] of positions 0 .. P.  Position i sees j
    with 0 <= i - j < size."""
    T, H, _ = q.shape
    out = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        i = first + t
        lo = max(0, i - size + 1)
        for h in range(H):
            s = (k[lo:i + 1, h] @ q[t, h]) * scale
            p = np.exp(s - s.max())
            out[t, h] = (p / p.sum()) @ v[lo:i + 1, h]
    return out


def latent_attention(h, w, c, eps, st, first):
    H, dim, rot, vdim, R = c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"]
    r = c["rot"]
    q = (rms_norm(h @ w("dq").T, w("dq.norm"), eps) @ w("uq").T).reshape(-1, H, dim + rot)
    down = h @ w("dkv").T
    latent, turned = rms_norm(down[:, :R], w("dkv.norm"), eps), down[:, R:].copy()
    for t in range(len(h)):
        q[t, :, dim:] = rotate_half(q[t, :, dim:], first + t, r["dims"], r["base"], r.get("scaling"))
        turned[t] = rotate_half(turned[t], first + t, r["dims"], r["base"], r.get("scaling"))
    st["c"] = latent = np.concatenate([st["c"], latent]) if "c" in st else latent
    st["r"] = turned = np.concatenate([st["r"], turned]) if "r" in st else turned
    k = np.concatenate([(latent @ w("uk").T).reshape(-1, H, dim), np.repeat(turned[:, None], H, axis=1)], axis=2)
    v = (latent @ w("uv").T).reshape(-1, H, vdim)
    o = window_attention(q, k, v, first, c["mask"]["size"], c["scale"]).reshape(len(h), -1)
    return (o * sigmoid(h @ w("g").T)) @ w("o").T


def linear_attention(S, q, k, v, decay):
    """One head: S [D, E], q and k [T, D], v [T, E], a constant decay."""
    S, o = S.copy(), np.zeros_like(v)
    for t in range(len(q)):
        S = decay * S + np.outer(k[t], v[t])
        o[t] = S.T @ q[t]
    return o, S


def lightning(h, w, c, eps, st):
    H, D, E = c["heads"], c["dim"], c["vdim"]
    q, k, v = (silu(h @ w(n).T).reshape(len(h), H, -1) for n in "qkv")
    S = st.get("S", np.zeros((H, D, E)))
    o, new = np.zeros_like(v), np.zeros_like(S)
    for i in range(H):
        o[:, i], new[i] = linear_attention(S[i], q[:, i], k[:, i], v[:, i], c["decay"][i])
    st["S"] = new
    o = rms_norm(o.reshape(len(h), H * E), w("norm"), eps)
    return (o * sigmoid(h @ w("g").T)) @ w("o").T


def mixer(kind, h, w, c, eps, st, first):
    if kind == "latent_attention":
        return latent_attention(h, w, c, eps, st, first)
    if kind == "lightning":
        return lightning(h, w, c, eps, st)
    raise ValueError(kind)


def glu(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def choose(z, top):
    """(experts with the largest scores, their scores), one token; the scores are not renormalised."""
    s = sigmoid(z)
    best = sorted(range(len(z)), key=lambda e: (-s[e], e))[:top]
    return best, s[best]


def experts(h, w, c):
    """Each token's chosen experts on the token scaled by their scores, and the shared expert on the token."""
    y = np.zeros_like(h)
    z = h @ w("router").T
    for t in range(len(h)):
        for e, s in zip(*choose(z[t], c["router"]["top"])):
            y[t] += glu(s * h[t], w(f"e{e}.gate"), w(f"e{e}.up"), w(f"e{e}.down"))
    if c.get("shared"):
        y = y + glu(h, w("shared.gate"), w("shared.up"), w("shared.down"))
    return y


class Sequence:
    """A sequence in progress: ``run(tokens)`` returns the logits of these tokens (and, if a list is given, appends the
    residual stream after every layer)."""

    def __init__(self, config, weights):
        self.c = config
        self.w = {n: np.asarray(t, F) for n, t in weights.items()}
        self.first = 0
        self.states = [{} for _ in config["layers"]]

    def run(self, tokens, layers=None):
        c, eps = self.c, self.c["norm"]["eps"]
        x = self.w["embed"][np.asarray(tokens, np.int64)]
        for i, layer in enumerate(c["layers"]):
            w = lambda n, p=f"l{i}.": self.w[p + n]
            y = mixer(layer["type"], rms_norm(x, w("norm1"), eps), lambda n: w("mix." + n), layer["mixer"], eps, self.states[i], self.first)
            x = x + rms_norm(y, w("norm1b"), eps)
            if layer["mlp"] is not None:
                y = experts(rms_norm(x, w("norm2"), eps), lambda n: w("mlp." + n), layer["mlp"])
                x = x + rms_norm(y, w("norm2b"), eps)
            if layers is not None:
                layers.append(x)
        self.first += len(tokens)
        return rms_norm(x, self.w["final.norm"], eps) @ self.w["head"].T
