"""Small configurations and random weights of the Lomozen design for the tests."""
import numpy as np
import torch

from khaosz_amd.hybrid import HybridConfig, HybridLM
from khaosz_amd.registry import load_tensors


def latent(heads=4, dim=24, rot_dim=8, vdim=40, q_rank=32, kv_rank=48, window=9, base=500.0, scale=0.4, dims=None, scaling="yarn"):
    if scaling == "yarn":
        scaling = {"factor": 4.0, "original": 64, "fast": 6.0, "slow": 1.5}
    rot = {"base": base, "dims": dims or rot_dim}
    if scaling:
        rot["scaling"] = scaling
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank,
                                                  "kv_rank": kv_rank, "mask": {"size": window}, "rot": rot, "scale": scale}}


def lightning(heads=3, dim=16, vdim=24, decay=None):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim,
                                           "decay": decay or [round(1 - 0.6 * 0.2 ** i, 6) for i in range(heads)]}}


def moe(experts=6, top=2, ff=40, shared=56):
    c = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}
    if shared:
        c["shared"] = {"ff": shared}
    return c


def layer(mixer, mlp="default"):
    return {**mixer, "mlp": moe() if mlp == "default" else mlp}


def config(layers, width=64, vocab=101, eps=1e-5):
    return {"architecture": "Lomozen", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width}


CASES = {
    # both mixers, unequal layers, one without a feed-forward
    "mixed": config([layer(lightning()), layer(latent()), layer(latent(2, 40, 16, 24, 48, 32, 70, 1e4, 0.15), moe(9, 1, 24, 16)),
                     layer(lightning(2, 40, 16, [0.5, 0.9995]), None)]),
    # nothing a multiple of 8: the kernels without alignment, no fused step
    "odd": config([layer(latent(3, 10, 6, 13, 11, 21, 17, 90.0, 0.3), moe(5, 3, 13, 9)), layer(lightning(5, 9, 7), moe(3, 1, 7, 5)),
                   layer(latent(1, 7, 2, 5, 9, 5, 40, 50.0, 0.5, scaling=None), None)], width=27, vocab=53),
    # heads and latents of a large model's layer; more heads than a matrix-core tile; several tiles of experts
    "wide": config([layer(latent(18, 128, 64, 128, 96, 512, 100, 5e4, 0.07), moe(40, 8, 32, 72)), layer(lightning(2, 128, 200, [0.97, 1.0]), moe(3, 3, 136, 24))],
                   width=72, vocab=64, eps=1e-6),
    # one head, a latent past the matrix-core decode, a state past the one-token kernel's, rotation of part of rot_dim, a window of 1
    "tall": config([layer(latent(1, 16, 24, 40, 16, 544, 1, 300.0, 0.3, dims=16)), layer(lightning(1, 24, 264, [0.8])),
                    layer(latent(2, 8, 8, 8, 8, 8, 4096, 1e3, 0.35), moe(2, 2, 8, 8))], width=40, vocab=48, eps=1e-3),
    # only attention, short windows: pages come back while a sequence runs
    "short": config([layer(latent(8, 64, 16, 64, 64, 64, 64, 700.0, 0.12)), layer(latent(5, 32, 32, 16, 40, 72, 33, 90.0, 0.2), moe(4, 1, 16, 8))],
                    width=48, vocab=80),
}


def weights(case, seed=0):
    """name -> float32 tensor, rounded to bf16 so that both number formats hold the same weights."""
    cfg = CASES[case] if isinstance(case, str) else case
    m = HybridLM(HybridConfig.from_dict(cfg), torch.float32, "cpu")
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name in sorted(m.tensors()):
        t = m.tensors()[name]
        r = torch.randn(t.shape, generator=g)
        if name == "embed":
            w = r
        elif t.dim() == 1:
            w = 1.0 + 0.3 * r
        else:
            w = r * (1.6 / t.shape[1] ** 0.5)
        out[name] = w.bfloat16().float()
    return out


def model(case, dtype, device="cuda:0", seed=0):
    cfg = CASES[case] if isinstance(case, str) else case
    m = HybridLM(HybridConfig.from_dict(cfg), dtype, device).eval()
    load_tensors(m, weights(case, seed))
    return m


def prompt(case, n, seed=1):
    cfg = CASES[case] if isinstance(case, str) else case
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()
