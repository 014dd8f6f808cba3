"""Small configurations and random weights of the hybrid decoder for the tests."""
import numpy as np
import torch

from khaosz_amd.hybrid import HybridConfig, HybridLM
from khaosz_amd.registry import load_tensors


def delta(heads=4, kv=2, dim=16, vdim=24, conv=3):
    return {"conv": conv, "dim": dim, "heads": heads, "kv_heads": kv, "vdim": vdim}


def attention(heads=4, kv=2, dim=24, vdim=40, window=9, rot=8, base=500.0, scale=0.4):
    return {"dim": dim, "heads": heads, "kv_heads": kv, "mask": {"size": window}, "rot": {"base": base, "dims": rot},
            "scale": scale, "vdim": vdim}


def mamba(heads=6, groups=2, state=24, vdim=16, conv=3, norm_groups=3):
    return {"conv": conv, "groups": groups, "heads": heads, "norm_groups": norm_groups, "state": state, "vdim": vdim}


def config(layers, width=64, vocab=101, eps=1e-5, mult=0.7, rank=(8, 16)):
    d = {"architecture": "Rudilix", "layers": layers, "norm": {"eps": eps}, "residual_mult": mult, "vocab": vocab, "width": width}
    shapes = {}
    for i, l in enumerate(layers):
        if l["type"] != "mamba2":
            p = f"l{i}.mix." + ("right." if l["type"] == "parallel" else "")
            shapes[p + "a1"], shapes[p + "g1"] = (rank[0], width), (rank[1], width)
    return d, shapes


def layer(kind, mixer, ff=96, limit=0.8):
    return {"type": kind, "mixer": mixer, "mlp": None if ff is None else {"ff": ff, "kind": "dense", "limit": limit}}


def parallel(left=None, right=None, ls=0.6, rs=1.3):
    return {"left": left or attention(), "left_scale": ls, "right": right or delta(), "right_scale": rs}


# sizes that differ in kind: several groups, unequal head counts, a layer without feed-forward, short and long windows
CASES = {
    "mixed": config([layer("parallel", parallel()), layer("mamba2", mamba(), ff=None), layer("channel_delta", delta(6, 3, 32, 8, 2), ff=40),
                     layer("mamba2", mamba(4, 1, 40, 24, 5, 1))]),
    # nothing a multiple of 8: the kernels without alignment, the products without the fused step
    "odd": config([layer("mamba2", mamba(3, 3, 10, 7, 2, 7), ff=33), layer("parallel", parallel(attention(3, 1, 10, 13, 17, 6), delta(3, 3, 9, 11, 4)), ff=20),
                   layer("channel_delta", delta(5, 1, 21, 5, 1), ff=None)], width=27, vocab=53, rank=(5, 3)),
    # heads wider than one tile, a convolution of one tap, a window longer than the tests' prompts, one repeated size
    "wide": config([layer("channel_delta", delta(2, 1, 136, 200, 4)), layer("parallel", parallel(attention(6, 1, 136, 144, 4096, 136, 1e4, 0.09), delta(2, 2, 72, 40, 1), 1.0, 1.0)),
                    layer("mamba2", mamba(2, 2, 144, 80, 1, 2), limit=7.0)], width=72, vocab=64, mult=1.0, eps=1e-6, rank=(24, 8)),
    # state columns past what the one-token kernels hold
    "tall": config([layer("channel_delta", delta(1, 1, 24, 264, 2)), layer("mamba2", mamba(1, 1, 16, 272, 4, 2), ff=24),
                    layer("parallel", parallel(attention(2, 2, 264, 296, 33, 264, 1e3, 0.06), delta(2, 1, 16, 40, 3)))], width=40, vocab=48),
    # several windows inside one page and one chunk
    "short": config([layer("parallel", parallel(attention(8, 4, 64, 64, 1, 64), delta(1, 1, 64, 64, 8))),
                     layer("parallel", parallel(attention(5, 1, 32, 128, 64, 2, 90.0, 0.3), delta(4, 4, 8, 16, 2)), ff=None)], width=48, vocab=80),
}


def weights(case, seed=0):
    """name -> float32 tensor, rounded to bf16 so that both number formats hold the same weights."""
    cfg, shapes = CASES[case] if isinstance(case, str) else case
    m = HybridLM(HybridConfig.from_dict(cfg, shapes), torch.float32, "cpu")
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, t in m.tensors().items():
        r = torch.randn(t.shape, generator=g)
        if name == "embed":
            w = r
        elif name.endswith(("norm1", "norm2")) or name == "final.norm":
            w = 0.3 * r
        elif name.endswith("norm"):
            w = 1.0 + 0.3 * r
        elif name.endswith("A_log"):
            w = 0.7 * r - 1.0
        elif name.endswith("dt_bias"):
            w = r - 1.0
        elif name.endswith((".conv", ".conv.b")):
            w = 0.5 * r
        elif name.endswith(".D") or t.dim() == 1:
            w = 0.5 * r
        else:
            w = r * (1.6 / t.shape[1] ** 0.5)
        out[name] = w.bfloat16().float()
    return out


def model(case, dtype, device="cuda:0", seed=0):
    cfg, shapes = CASES[case] if isinstance(case, str) else case
    m = HybridLM(HybridConfig.from_dict(cfg, shapes), dtype, device).eval()
    load_tensors(m, weights(case, seed))
    return m


def prompt(case, n, seed=1):
    cfg, _ = CASES[case] if isinstance(case, str) else case
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()
