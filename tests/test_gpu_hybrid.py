"""The hybrid decoder on the GPU against its plain restatement (oracle/hybrid.py): every mechanism alone, then whole
models -- prompts, portions, single tokens, batches of unequal sequences, reused slots and pages, window edges, long
decoding, greedy generation."""
import numpy as np
import pytest
import torch

from khaosz_amd import Engine, seq_ops
from khaosz_amd.mixers import rotary_pairs
from khaosz_amd.sampling import Sampler
from khaosz_amd.seq_ops import Batch, WindowAttnSpec
from oracle import hybrid as plain

import hybrid_cases as hc

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = [torch.float32, torch.bfloat16]


def rnd(*shape, seed=0, scale=1.0):
    return (torch.randn(shape, generator=torch.Generator().manual_seed(seed)) * scale).bfloat16().float()


def f64(t):
    return t.detach().double().cpu().numpy()


def batch(pos, slots, S, table=None):
    B = len(pos)
    t = torch.zeros((B, 1), dtype=torch.int64) if table is None else table
    return Batch(torch.tensor(pos, dtype=torch.int32, device=DEV), torch.tensor(slots, dtype=torch.int32, device=DEV), t.to(DEV), B, S)


def close(got, want, dtype, rel=None, low=1.5e-2):
    """Relative to the want's root mean square: fp32 within accumulation order everywhere; bf16 within a few roundings
    in the root mean square, with room for single elements where a softmax is nearly a tie."""
    got, want = f64(got) if torch.is_tensor(got) else got, np.asarray(want)
    assert got.shape == want.shape, (got.shape, want.shape)
    d, size = got - want, np.sqrt((want ** 2).mean()) + 1e-30
    if dtype == torch.float32:
        assert np.abs(d).max() / size < (rel or 6e-5), np.abs(d).max() / size
    else:
        assert np.sqrt((d ** 2).mean()) / size < low and np.abs(d).max() / size < 0.3, (np.sqrt((d ** 2).mean()) / size, np.abs(d).max() / size)


# ------------------------------------------------------------------------------------------------ rows
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,K", [(1, 64), (5, 27), (3, 2048), (2, 5001)])
def test_add_and_norm(dtype, M, K):
    x, y, w = rnd(M, K, seed=1), rnd(M, K, seed=2), rnd(K, seed=3, scale=0.3)
    xd = x.to(DEV)
    h = seq_ops.add_rmsnorm(xd, y.to(DEV, dtype), 0.37, w.to(DEV), 1e-3, dtype)
    want = f64(x) + 0.37 * f64(y)
    close(xd, want, torch.float32)
    close(h, plain.rms_norm_plus_one(want, f64(w), 1e-3), dtype)
    assert seq_ops.add_rmsnorm(xd, None, 1.0, None, 0.0, dtype, norm=False) is None
    close(xd, want, torch.float32)


def test_epsilon_sits_inside_the_root():
    x = torch.full((1, 32), 1e-3, device=DEV)
    h = seq_ops.add_rmsnorm(x, None, 1.0, torch.zeros(32, device=DEV), 1e-6, torch.float32)
    assert torch.allclose(h, torch.full_like(h, 1e-3 / (2e-6) ** 0.5), rtol=1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
def test_embedding(dtype):
    t = rnd(9, 20)
    got = seq_ops.embed(torch.tensor([3, 0, 8, 3, 9, -1], device=DEV), t.to(DEV, dtype))
    want = torch.cat([t[[3, 0, 8, 3]], torch.zeros(2, 20)])
    assert got.dtype == torch.float32 and torch.equal(got.cpu(), want)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("F", [40, 33])
def test_clamped_glu(dtype, F):
    gu = rnd(7, 2 * F, scale=3.0)
    gu[0, 0], gu[0, 1], gu[0, F], gu[0, F + 1] = 50.0, -50.0, 50.0, -50.0
    g, u = np.minimum(f64(gu[:, :F]), 0.9), np.clip(f64(gu[:, F:]), -0.9, 0.9)
    close(seq_ops.clamped_glu(gu.to(DEV, dtype), 0.9), g * plain.sigmoid(1.702 * g) * (u + 1), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("K,groups", [(48, 1), (48, 3), (35, 7), (1280, 2)])
def test_gated_group_norm(dtype, K, groups):
    y, z, w = rnd(4, K, seed=1), rnd(4, K + 5, seed=2), rnd(K, seed=3)
    out = torch.empty((4, K + 3), dtype=dtype, device=DEV)
    seq_ops.gated_group_norm(y.to(DEV), z.to(DEV, dtype), 5, w.to(DEV), 1e-4, groups, out[:, 3:])
    v = (f64(y) * plain.silu(f64(z[:, 5:]))).reshape(4, groups, -1)
    close(out[:, 3:], plain.rms(v, 1e-4).reshape(4, K) * f64(w), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,E", [(3, 24), (2, 5), (1, 200)])
def test_head_norm_and_gate(dtype, H, E):
    o, gate, w = rnd(5, H, E, seed=1), rnd(5, H * E, seed=2), rnd(E, seed=3)
    out = torch.empty((5, H * E), dtype=dtype, device=DEV)
    seq_ops.head_norm_gate(o.to(DEV), gate.to(DEV, dtype), w.to(DEV), 1e-4, 1.3, out)
    close(out, 1.3 * (plain.rms(f64(o), 1e-4) * f64(w) * plain.sigmoid(f64(gate)).reshape(5, H, E)).reshape(5, -1), dtype)


# ------------------------------------------------------------------------------------------------ matrix-vector products
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,N,K", [(1, 30, 24), (3, 101, 512), (8, 64, 2064), (1, 4100, 200), (2, 8200, 48), (5, 16, 4096)])
def test_matrix_vector_products(dtype, M, N, K):
    x, gain, w = rnd(M, K, seed=1), rnd(K, seed=2, scale=0.3), rnd(N, K, seed=3, scale=K ** -0.5)
    bias, res, z = rnd(N, seed=4), rnd(M, N, seed=5), rnd(M, K + 8, seed=6)
    xd, gd, wd = x.to(DEV), gain.to(DEV), w.to(DEV, dtype)
    kept = torch.float32 if M == 1 else dtype  # several rows are kept in the activations' format
    h = plain.rms_norm_plus_one(f64(x), f64(gain), 1e-5)
    close(seq_ops.norm_gemv(xd, gd, 1e-5, wd, bias.to(DEV)), h @ f64(w).T + f64(bias), dtype)
    close(seq_ops.norm_gemv_f32(xd, gd, 1e-5, wd), h @ f64(w).T, kept)
    if N % 2 == 0:
        F = N // 2
        g, u = np.minimum(h @ f64(w[:F]).T, 0.6), np.clip(h @ f64(w[F:]).T, -0.6, 0.6)
        close(seq_ops.norm_gemv_glu(xd, gd, 1e-5, wd, 0.6), g * plain.sigmoid(1.702 * g) * (u + 1), dtype)
    rd = res.to(DEV)
    seq_ops.gemv_residual(x.to(DEV, dtype), wd, 0.7, rd)
    close(rd, f64(res) + 0.7 * (f64(x) @ f64(w).T), torch.float32)
    for groups in (1, 4):
        rd = res.to(DEV)
        seq_ops.gated_norm_gemv_residual(xd, z.to(DEV, dtype), 8, gd, 1e-5, groups, wd, 0.7, rd)
        v = plain.rms((f64(x) * plain.silu(f64(z[:, 8:]))).reshape(M, groups, -1), 1e-5).reshape(M, K) * f64(gain)
        close(rd, f64(res) + 0.7 * (v @ f64(w).T), kept)


# ------------------------------------------------------------------------------------------------ convolution
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps", [1, 2, 4, 7])
def test_convolution_carries_its_inputs(dtype, taps):
    C, T = 37, 30
    x, w, bias = rnd(T, C + 3, seed=1), rnd(C, taps, seed=2), rnd(C, seed=3)
    xd = x.to(DEV, dtype)
    want, _ = plain.causal_conv(f64(x[:, 3:]), f64(w), f64(bias))
    want = plain.silu(want)
    ring = torch.full((3, taps, C), 99.0, dtype=dtype, device=DEV)  # an earlier owner's content
    for cuts in ([30], [2, 3, 2, 9, 1, 1, 12], [1] * 30):
        at, out = 0, []
        for n in cuts:
            b = batch([at], [1], n)
            out.append(seq_ops.conv_silu(xd[at:at + n], 3, w.to(DEV), bias.to(DEV), ring, b))
            seq_ops.conv_push(xd[at:at + n], 3, C, taps, ring, b)
            at += n
        close(torch.cat(out), want, torch.float32)
    assert bool((ring[[0, 2]] == 99).all())


# ------------------------------------------------------------------------------------------------ recurrences
DELTA_SIZES = [(1, 1, 16, 16), (4, 2, 32, 24), (3, 1, 20, 37), (2, 2, 128, 64), (2, 1, 136, 200), (6, 3, 10, 5), (1, 1, 256, 256)]


@pytest.mark.parametrize("H,G,D,E", DELTA_SIZES)
def test_delta_rule_scan(H, G, D, E):
    T = 45
    q, k = plain.unit(f64(rnd(T, G, D, seed=1))) * D ** -0.5, plain.unit(f64(rnd(T, G, D, seed=2)))
    v, beta = f64(rnd(T, H, E, seed=3)), plain.sigmoid(f64(rnd(T, H, seed=4, scale=2.0)))
    decay = np.exp(-np.exp(f64(rnd(T, H, D, seed=5, scale=2.0))))  # from 1 down to the smallest floats
    k[20], k[21] = k[19], k[19]                                    # the same key written three times in a row
    want = np.stack([plain.delta_rule(np.zeros((D, E)), q[:, h // (H // G)], k[:, h // (H // G)], v[:, h], decay[:, h], beta[:, h])[0]
                     for h in range(H)], 1)
    dev = [torch.tensor(a, dtype=torch.float32, device=DEV).contiguous() for a in (q, k, v, decay, beta)]
    for cuts in ([45], [16, 29], [2, 17, 3, 16, 7], [1] * 45):
        state, at, out = torch.full((2, H, E, D), 7.0, device=DEV), 0, []
        for n in cuts:
            out.append(seq_ops.delta_scan(*[a[at:at + n].contiguous() for a in dev], state, batch([at], [1], n)))
            at += n
        close(torch.cat(out), want, torch.float32)
        assert bool((state[0] == 7).all())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,E,taps", [(4, 2, 24, 40, 3), (3, 3, 10, 7, 4), (2, 1, 136, 200, 1)])
def test_delta_inputs(dtype, H, G, D, E, taps):
    T, C = 9, 2 * G * D + H * E
    proj, raw, w = rnd(T, C + H + 4, seed=1), rnd(T, H * D, seed=2, scale=3.0), rnd(C, taps, seed=3)
    a_log, dt = rnd(H, seed=4), rnd(H * D, seed=5)
    raw[0, 0] = 100.0                                              # softplus of a large argument is the argument
    got = seq_ops.delta_prep(proj.to(DEV, dtype), 4, raw.to(DEV, dtype), 4 + C, w.to(DEV), torch.zeros((1, taps, C), dtype=dtype, device=DEV),
                             a_log.to(DEV), dt.to(DEV), H, G, D, E, batch([0], [0], T))
    act = plain.silu(plain.causal_conv(f64(proj[:, 4:4 + C]), f64(w))[0])
    close(got[0], plain.unit(act[:, :G * D].reshape(T, G, D)) * D ** -0.5, torch.float32)
    close(got[1], plain.unit(act[:, G * D:2 * G * D].reshape(T, G, D)), torch.float32)
    close(got[2], act[:, 2 * G * D:].reshape(T, H, E), torch.float32)
    close(got[3], np.exp(-np.exp(f64(a_log))[:, None] * plain.softplus(f64(raw) + f64(dt)).reshape(T, H, D)), torch.float32)
    close(got[4], plain.sigmoid(f64(proj[:, 4 + C:])), torch.float32)


SSD_SIZES = [(1, 1, 16, 16), (6, 2, 24, 16), (3, 3, 10, 7), (4, 1, 128, 64), (2, 2, 144, 80), (2, 1, 256, 256)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,N,P", SSD_SIZES)
def test_ssd_scan(dtype, H, G, N, P):
    T, C = 45, H * P + 2 * G * N
    xbc, dt_raw = rnd(T, C, seed=1), rnd(T, H + 2, seed=2, scale=2.0)
    a_log, dtb, skip = rnd(H, seed=3), rnd(H, seed=4), rnd(H, seed=5)
    dt_raw[7, 2] = 60.0                                            # forgets everything
    dt = plain.softplus(f64(dt_raw[:, 2:]) + f64(dtb))
    a = f64(xbc)
    x, B, Cc = a[:, :H * P].reshape(T, H, P), a[:, H * P:H * P + G * N].reshape(T, G, N), a[:, H * P + G * N:].reshape(T, G, N)
    want = np.stack([plain.ssd(np.zeros((N, P)), x[:, h], B[:, h // (H // G)], Cc[:, h // (H // G)], dt[:, h], f64(a_log)[h], f64(skip)[h])[0]
                     for h in range(H)], 1).reshape(T, -1)
    xd, pd = xbc.to(DEV), dt_raw.to(DEV, dtype)
    for cuts in ([45], [16, 29], [2, 17, 3, 16, 7], [1] * 45):
        state, at, out = torch.full((2, H, P, N), 7.0, device=DEV), 0, []
        for n in cuts:
            out.append(seq_ops.ssd_scan(xd[at:at + n].contiguous(), pd[at:at + n], 2, dtb.to(DEV), a_log.to(DEV), skip.to(DEV), state,
                                        H, G, N, P, batch([at], [1], n)))
            at += n
        close(torch.cat(out), want, torch.float32)
        assert bool((state[0] == 7).all())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,E,taps,strength", [(1, 1, 16, 16, 1, 1.0), (4, 2, 32, 24, 3, 2.0), (3, 1, 20, 37, 4, 3.0), (2, 2, 128, 64, 4, 1.0),
                                                   (2, 1, 100, 200, 2, 4.5), (1, 1, 64, 128, 4, 6.0)])
def test_delta_rule_in_chunks(dtype, H, G, D, E, taps, strength):
    """Weak to very strong decays (down to e^-hundreds a token, where a factored exponent would overflow), cut anywhere."""
    T, C = 270, 2 * G * D + H * E
    proj, raw, w = rnd(T, C + H + 4, seed=1), rnd(T, H * D, seed=2, scale=strength), rnd(C, taps, seed=3)
    a_log, dt = rnd(H, seed=4, scale=0.5 * strength), rnd(H * D, seed=5)
    raw[40:43] = 90.0                                              # forgets everything, in the middle of a chunk
    raw[100:140] = -20.0                                           # forgets nothing
    proj[60:64, 4:4 + C] = proj[59, 4:4 + C]                       # equal keys around a chunk's edge
    beta = plain.sigmoid(f64(proj[:, 4 + C:]))
    act = plain.silu(plain.causal_conv(f64(proj[:, 4:4 + C]), f64(w))[0])
    q, k = plain.unit(act[:, :G * D].reshape(T, G, D)) * D ** -0.5, plain.unit(act[:, G * D:2 * G * D].reshape(T, G, D))
    v = act[:, 2 * G * D:].reshape(T, H, E)
    decay = np.exp(-np.exp(f64(a_log))[:, None] * plain.softplus(f64(raw) + f64(dt)).reshape(T, H, D))
    run = [plain.delta_rule(np.zeros((D, E)), q[:, h // (H // G)], k[:, h // (H // G)], v[:, h], decay[:, h], beta[:, h]) for h in range(H)]
    want, last = np.stack([o for o, _ in run], 1), np.stack([S.T for _, S in run])
    pd, rd = proj.to(DEV, dtype), raw.to(DEV, dtype)
    for cuts in ([270], [64, 128, 78], [65, 2, 130, 63, 10]):
        state, at, out = torch.full((2, H, E, D), 7.0, device=DEV), 0, []
        ring = torch.full((2, taps, C), 99.0, dtype=dtype, device=DEV)
        for n in cuts:
            b = batch([at], [1], n)
            out.append(seq_ops.delta_chunked(pd[at:at + n], 4, rd[at:at + n], 4 + C, w.to(DEV), ring, a_log.to(DEV), dt.to(DEV), state, H, G, D, E, b))
            seq_ops.conv_push(pd[at:at + n], 4, C, taps, ring, b)
            at += n
        close(torch.cat(out), want, torch.float32)
        close(state[1], last, torch.float32)
        assert bool((state[0] == 7).all())
    # two sequences in one call, one of them in the middle of its text
    b = batch([0, 100], [1, 0], 100)
    two = torch.cat([pd[:100], pd[100:200]])
    state[0].copy_(torch.zeros_like(state[0]))
    one = seq_ops.delta_chunked(pd[:100], 4, rd[:100], 4 + C, w.to(DEV), ring, a_log.to(DEV), dt.to(DEV), state, H, G, D, E, batch([0], [0], 100))
    seq_ops.conv_push(pd[:100], 4, C, taps, ring, batch([0], [0], 100))
    both = seq_ops.delta_chunked(two, 4, torch.cat([rd[:100], rd[100:200]]), 4 + C, w.to(DEV), ring, a_log.to(DEV), dt.to(DEV), state, H, G, D, E, b)
    assert torch.equal(both[:100], one)
    close(both, want[:200], torch.float32)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,N,P,taps", [(1, 1, 16, 16, 1), (6, 2, 24, 16, 3), (3, 3, 10, 7, 4), (4, 1, 128, 64, 4), (2, 2, 100, 80, 2), (2, 1, 64, 200, 4)])
def test_ssd_in_chunks(dtype, H, G, N, P, taps):
    T, C = 270, H * P + 2 * G * N
    proj, w, bias = rnd(T, 3 + C + H, seed=1), rnd(C, taps, seed=2), rnd(C, seed=6)
    a_log, dtb, skip = rnd(H, seed=3), rnd(H, seed=4), rnd(H, seed=5)
    proj[40, 3 + C:], proj[100:140, 3 + C:] = 60.0, -12.0          # forgets everything; hardly moves
    act = plain.silu(plain.causal_conv(f64(proj[:, 3:3 + C]), f64(w), f64(bias))[0])
    dt = plain.softplus(f64(proj[:, 3 + C:]) + f64(dtb))
    x, B, Cc = act[:, :H * P].reshape(T, H, P), act[:, H * P:H * P + G * N].reshape(T, G, N), act[:, H * P + G * N:].reshape(T, G, N)
    run = [plain.ssd(np.zeros((N, P)), x[:, h], B[:, h // (H // G)], Cc[:, h // (H // G)], dt[:, h], f64(a_log)[h], f64(skip)[h]) for h in range(H)]
    want, last = np.stack([y for y, _ in run], 1).reshape(T, -1), np.stack([S.T for _, S in run])
    pd = proj.to(DEV, dtype)
    for cuts in ([270], [64, 128, 78], [65, 2, 130, 63, 10]):
        state, at, out = torch.full((2, H, P, N), 7.0, device=DEV), 0, []
        ring = torch.full((2, taps, C), 99.0, dtype=dtype, device=DEV)
        for n in cuts:
            b = batch([at], [1], n)
            out.append(seq_ops.ssd_chunked(pd[at:at + n], 3, 3 + C, w.to(DEV), bias.to(DEV), ring, dtb.to(DEV), a_log.to(DEV), skip.to(DEV),
                                           state, H, G, N, P, b))
            seq_ops.conv_push(pd[at:at + n], 3, C, taps, ring, b)
            at += n
        close(torch.cat(out), want, torch.float32)
        close(state[1], last, torch.float32)
        assert bool((state[0] == 7).all())


# ------------------------------------------------------------------------------------------------ windowed attention
ATTN = [  # H, G, D, E, window, rot, T
    (4, 2, 24, 40, 9, 8, 70), (3, 1, 10, 13, 17, 6, 40), (6, 3, 128, 128, 64, 64, 200), (8, 1, 64, 64, 65, 64, 150),
    (4, 4, 136, 256, 128, 0, 300), (5, 1, 256, 72, 1, 256, 130), (2, 2, 32, 200, 5000, 32, 210), (7, 1, 96, 16, 63, 2, 140)]


class Attn:
    """One attention with raw projections planted so that single keys stand out: query i points at key i - window + 1
    (the last one inside) for one half of the queries and at key i - window (just outside) for the other."""

    def __init__(self, dtype, H, G, D, E, window, rot, T, page=64, pages=None):
        self.spec = WindowAttnSpec(H, G, D, E, window, 0.9, rot, 1e-5)
        self.T, self.W, self.dtype = T, H * D + G * D + G * E + H, dtype
        self.o = (0, H * D, H * D + G * D, H * D + G * D + G * E)
        proj = rnd(T, self.W, seed=7, scale=0.5)
        plain_dims = list(range(rot, D))  # not rotated: a match there holds at any distance
        for i in range(T):
            j = i - window + (1 if i % 2 else 0)
            if plain_dims and 0 <= j < T:
                for h in range(H):
                    proj[i, h * D + rot:(h + 1) * D] = 4 * proj[j, H * D + (h // (H // G)) * D + rot:H * D + (h // (H // G) + 1) * D]
        self.proj = proj.bfloat16().float()
        self.qn, self.kn = rnd(D, seed=8, scale=0.2) + 1, rnd(D, seed=9, scale=0.2) + 1
        self.cs = rotary_pairs(rot, 8192 if T > 4000 else 1024, 700.0).to(DEV)
        n = (T + page - 1) // page
        self.table = torch.randperm(n + 2, generator=torch.Generator().manual_seed(3))[:n].view(1, n)
        self.kc = torch.full((n + 2, page, G, D), 50.0, dtype=dtype, device=DEV)
        self.vc = torch.full((n + 2, page, G, E), 50.0, dtype=dtype, device=DEV)

    def want(self, scale=1.0):
        s, p = self.spec, f64(self.proj)
        q, k, v = (p[:, a:b].reshape(self.T, n, -1) for a, b, n in ((self.o[0], self.o[1], s.H), (self.o[1], self.o[2], s.G), (self.o[2], self.o[3], s.G)))
        q, k = plain.rms(q, s.eps) * f64(self.qn), plain.rms(k, s.eps) * f64(self.kn)
        q = np.stack([plain.rotate(q[t], t, s.rot, 700.0) if s.rot else q[t] for t in range(self.T)])
        k = np.stack([plain.rotate(k[t], t, s.rot, 700.0) if s.rot else k[t] for t in range(self.T)])
        o = plain.window_attention(q, k, v, 0, s.window, s.scale) * plain.sigmoid(p[:, self.o[3]:])[:, :, None]
        return scale * o.reshape(self.T, -1)

    def portion(self, at, n, scale=1.0, simple=False, decode=False):
        b, s = batch([at], [0], n, self.table), self.spec
        p = self.proj[at:at + n].to(DEV, self.dtype)
        out = torch.empty((n, s.H * s.E), dtype=self.dtype, device=DEV)
        args = (self.qn.to(DEV), self.kn.to(DEV), self.cs, self.kc, self.vc)
        if decode:
            seq_ops.attn_decode(p, *self.o, *args, scale, s, b, out)
        else:
            q = seq_ops.attn_prep(p, *self.o[:3], *args, s, b)
            seq_ops.attn_window(q, self.kc, self.vc, p, self.o[3], scale, s, b, out, simple)
        return out


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", ATTN, ids=str)
def test_windowed_attention(dtype, sizes):
    T = sizes[-1]
    want = Attn(dtype, *sizes).want(0.8)
    tol = 1e-4
    for simple in (False, True):
        for cuts in ([T], [2, 3, 61, T - 66], [63, 1, 2, 64][:4] if T <= 130 else [63, 1, 2, T - 66]):
            a, at, out = Attn(dtype, *sizes), 0, []
            for n in cuts:
                n = min(n, T - at)
                if n > 0:
                    out.append(a.portion(at, n, 0.8, simple))
                    at += n
            if at < T:
                out.append(a.portion(at, T - at, 0.8, simple))
            close(torch.cat(out), want, dtype, tol)
    if sizes[2] % 8 == 0 and sizes[3] % 8 == 0:
        a = Attn(dtype, *sizes)
        first = T // 3
        out = [a.portion(0, first, 0.8)] + [a.portion(t, 1, 0.8, decode=True) for t in range(first, T)]
        close(torch.cat(out), want, dtype, tol)
        # from the very first token on
        a = Attn(dtype, *sizes)
        close(torch.cat([a.portion(t, 1, 0.8, decode=True) for t in range(min(T, 70))]), want[:70], dtype, tol)


# ------------------------------------------------------------------------------------------------ whole models
def oracle_logits(case, ids):
    cfg, _ = hc.CASES[case]
    return plain.Sequence(cfg, {n: t.numpy() for n, t in hc.weights(case).items()}).run(ids)


def check(got, want, dtype):
    d = np.asarray(got, np.float64) - want
    d -= d.mean(-1, keepdims=True)
    err = np.sqrt((d ** 2).mean(-1)) / want.std()  # by position
    assert err.max() < (2e-5 if dtype == torch.float32 else 0.2), (err.max(), int(err.argmax()))
    if dtype == torch.bfloat16 and len(err) > 3:
        assert np.sqrt((err ** 2).mean()) < 4e-2, err


def feed(e, h, ids, cuts):
    at, out = 0, []
    for n in cuts:
        out.append(e.step([h], [ids[at:at + n]]).float().cpu().numpy())
        at += n
    assert at == len(ids)
    return np.concatenate(out)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", list(hc.CASES))
def test_model_whole_in_portions_and_by_token(case, dtype):
    T = 150
    ids = hc.prompt(case, T)
    want = oracle_logits(case, ids)
    e = Engine(hc.model(case, dtype), T, 1)
    for cuts in ([T], [64, 64, 22], [100, 50], [2] * 75, [7, 2, 3, 50, 1, 1, 1, 63, 22], [1] * T, [100] + [1] * 50):
        h = e.open()  # the same slot and pages every time
        check(feed(e, h, ids, cuts), want, dtype)
        e.close(h)


@pytest.mark.parametrize("dtype", DTYPES)
def test_layers_of_the_float_model(dtype):
    case = "mixed"
    ids, layers = hc.prompt(case, 40), []
    cfg, _ = hc.CASES[case]
    plain.Sequence(cfg, {n: t.numpy() for n, t in hc.weights(case).items()}).run(ids, layers)
    m = hc.model(case, dtype)
    c = Engine(m, 64).cache
    h = c.open()
    c.reserve([h], 40)
    w = np.empty(c.words(1, 40), np.int64)
    c.pack([h], [ids], w)
    got = []
    with torch.inference_mode():
        m(*c.unpack(torch.from_numpy(w).to(DEV), 1, 40), c.state, None, got)
    for a, b in zip(got, layers):
        close(a, b, dtype, low=3e-2)


@pytest.mark.parametrize("dtype", DTYPES)
def test_only_wanted_rows_are_returned(dtype):
    case, T = "mixed", 30
    ids = hc.prompt(case, T)
    want = oracle_logits(case, ids)
    e = Engine(hc.model(case, dtype), T)
    for rows in ([0], [29], [3, 2, 17], list(range(5, 25)), []):
        h = e.open()
        got = e.step([h], [ids], rows).cpu().numpy()
        assert got.shape == (len(rows), want.shape[1])
        if rows:
            check(got, want[rows], dtype)
        e.close(h)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", ["mixed", "odd", "short"])
def test_unequal_sequences_share_steps(case, dtype):
    """Prompts of different lengths, then single tokens of all of them in one step, some ending and others starting in
    their slots and pages meanwhile: every sequence as if alone."""
    lens, total = [5, 70, 33], 90
    seqs = [hc.prompt(case, total, seed=20 + i) for i in range(4)]
    wants = [oracle_logits(case, s) for s in seqs]
    e = Engine(hc.model(case, dtype), 4 * total, 4)
    hs = [e.open() for _ in lens]
    at = list(lens)
    for i, h in enumerate(hs):
        check(e.step([h], [seqs[i][:lens[i]]]).cpu().numpy(), wants[i][:lens[i]], dtype)
    for step in range(20):
        order = [2, 0, 1] if step % 3 else [1, 0, 2]
        got = e.step([hs[i] for i in order], [[seqs[i][at[i]]] for i in order]).cpu().numpy()
        for g, i in zip(got, order):
            check(g[None], wants[i][at[i]][None], dtype)
            at[i] += 1
    e.close(hs[1])
    fresh = e.open()  # takes slot and pages of the one that ended
    check(e.step([fresh], [seqs[3][:40]]).cpu().numpy(), wants[3][:40], dtype)
    for t in range(40, 50):
        got = e.step([hs[0], fresh], [[seqs[0][at[0]]], [seqs[3][t]]]).cpu().numpy()
        check(got, np.stack([wants[0][at[0]], wants[3][t]]), dtype)
        at[0] += 1


def test_portions_of_several_sequences_at_once():
    case, dtype = "mixed", torch.float32
    seqs = [hc.prompt(case, 60, seed=30 + i) for i in range(3)]
    wants = [oracle_logits(case, s) for s in seqs]
    e = Engine(hc.model(case, dtype), 200, 3)
    hs = [e.open() for _ in seqs]
    e.step([hs[1]], [seqs[1][:9]])
    got = e.step([hs[2], hs[1], hs[0]], [seqs[2][:20], seqs[1][9:29], seqs[0][:20]]).cpu().numpy()
    check(got, np.concatenate([wants[2][:20], wants[1][9:29], wants[0][:20]]), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_replayed_step_is_the_eager_step(dtype):
    case = "mixed"
    ids = hc.prompt(case, 60)
    m = hc.model(case, dtype)
    eager, graph = Engine(m, 64, graphs=False), Engine(m, 64)
    a, b = eager.open(), graph.open()
    for t in range(60):
        x, y = eager.step([a], [[ids[t]]]).clone(), graph.step([b], [[ids[t]]]).clone()
        assert torch.equal(x, y), t
    assert graph._graphs and not eager._graphs


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_returns_the_pages_behind_the_window(dtype):
    """More tokens than the cache has pages: every layer's window is short, so pages come back on the way."""
    case, T = "short", 420
    ids = hc.prompt(case, T)
    want = oracle_logits(case, ids)
    e = Engine(hc.model(case, dtype), 448)
    h = e.open()
    got = []
    for t in range(T):
        got.append(e.step([h], [[ids[t]]]).cpu().numpy())
        assert (e.cache.table >= 0).sum() <= 2
    check(np.concatenate(got), want, dtype)


def test_far_prompt_through_the_recurrences():
    """A prompt of many scan chunks and key blocks, cut in the middle of both."""
    case, T = "mixed", 700
    ids = hc.prompt(case, T)
    want = oracle_logits(case, ids)
    e = Engine(hc.model(case, torch.float32), T)
    for cuts in ([T], [333, 367], [600] + [1] * 100):
        h = e.open()
        check(feed(e, h, ids, cuts), want, torch.float32)
        e.close(h)


@pytest.mark.parametrize("case", ["mixed", "odd"])
def test_greedy_generation_follows_the_oracle(case):
    cfg, _ = hc.CASES[case]
    w = {n: t.numpy() for n, t in hc.weights(case).items()}
    prompts = [hc.prompt(case, n, seed=40 + n) for n in (3, 1, 20, 11, 7)]

    def alone(p, n):
        s, out = plain.Sequence(cfg, w), []
        z = s.run(p)[-1]
        for _ in range(n):
            out.append(int(z.argmax()))
            z = s.run([out[-1]])[0]
        return out
    want = [alone(p, 25) for p in prompts]
    e = Engine(hc.model(case, torch.float32), 150, 3)
    assert e.generate(prompts, 25, Sampler()) == want
    assert len(e.cache.slots) == 3 and (e.cache.table < 0).all()
    assert Engine(hc.model(case, torch.float32), 60).generate(prompts[:2], 25) == want[:2]


def test_sampling_is_repeatable():
    m = hc.model("mixed", torch.bfloat16)
    p = [hc.prompt("mixed", 5)]
    draw = lambda seed: Engine(m, 64).generate(p, 20, Sampler(0.9, 20, 0.95, seed))
    assert draw(1) == draw(1) and draw(1) != draw(2)


def test_trace_runner(tmp_path):
    import json
    import os
    import subprocess
    import sys

    from safetensors.torch import save_file
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    case = "mixed"
    cfg, _ = hc.CASES[case]
    (tmp_path / "m").mkdir()
    (tmp_path / "m" / "config.json").write_text(json.dumps(cfg))
    save_file({n: t.bfloat16().contiguous() for n, t in hc.weights(case).items()}, str(tmp_path / "m" / "model.safetensors"))
    a, b = hc.prompt(case, 40, 50), hc.prompt(case, 12, 51)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:30], "want": [29, 3]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[30:38], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[38:39], "want": [0]}], "end": []},
             {"step": 3, "entries": [{"id": "a", "tokens": a[39:], "want": [0]}], "end": ["a"]},
             {"step": 4, "entries": [{"id": "b", "tokens": b, "want": list(range(12))}], "end": ["b"]}]
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", "float32",
                        "--out", str(tmp_path), "--max-tokens", "40"], input="\n".join(map(json.dumps, steps)), text=True,
                       capture_output=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(5)]
    read = lambda i: np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(-1, cfg["vocab"])
    wa, wb = oracle_logits(case, a), oracle_logits(case, b)
    check(read(0), wa[[29, 3]], torch.float32)
    assert not (tmp_path / "1.f32").exists()
    check(np.concatenate([read(2), read(3)]), wa[38:], torch.float32)
    check(read(4), wb, torch.float32)
