"""Token mixers of the hybrid decoders beside ``block.GQA``: sliding-window attention, the gated delta rule
with one decay per key channel, the Mamba-2 state-space mixer, latent attention, linear attention with a constant decay per
head, and their composition side by side; and the feed-forwards, dense and routed.

A mixer reads columns of one fused input projection and writes columns of the input of one fused output
projection; ``MixerBlock`` owns both matrices.  So mixers that read the same input side by side cost one
product in front and one behind, whatever they are.  Each mixer has two forms: ``prompt`` for any number of
new tokens per sequence (convolution, scan, norm as separate launches around the vendor's matrix products)
and ``step`` for one new token per sequence (everything between the two projections in one launch).

Weights are kept under the names their checkpoint uses; ``tensors()`` of every module maps those names to
(views of) its parameters.
"""
from __future__ import annotations

import math
from typing import Any, Dict, List, NamedTuple, Optional, Sequence, Tuple

import torch
import torch.nn as nn
import torch.nn.functional as F
from torch import Tensor

from . import seq_ops
from .block import PagedKV
from .seq_ops import Batch, LatentSpec, Routed, Stream, WindowAttnSpec


def _round8(n: int) -> int:
    return (n + 7) // 8 * 8


def _param(*shape, dtype=torch.float32, device=None) -> nn.Parameter:
    return nn.Parameter(torch.zeros(shape, dtype=dtype, device=device), requires_grad=False)


class Branch(NamedTuple):
    """What a mixer or feed-forward leaves to be added to the stream: rows ``y [M, width]`` (or none), each token's routed
    rows, and the weight of a norm that the sum of them passes first."""
    y: Optional[Tensor]
    routed: Optional[Routed] = None
    post: Optional[Tensor] = None

    def rows(self, want: Tensor) -> "Branch":
        routed = self.routed
        if routed is not None:
            routed = Routed(routed.rows, routed.slots[want].contiguous())
        return Branch(None if self.y is None else self.y[want], routed, self.post)


def yarn(inv: Tensor, base: float, scaling: Dict[str, Any]) -> Tuple[Tensor, float]:
    """YaRN (Peng et al., "YaRN: Efficient Context Window Extension of Large Language Models"): frequencies of dimensions
    that turn fewer than ``slow`` times within ``original`` positions are divided by ``factor``, those that turn more than
    ``fast`` times are kept, with a ramp between; cosines and sines grow by the returned factor."""
    dims, factor = 2 * len(inv), float(scaling["factor"])

    def dim_of(turns: float) -> float:
        return dims * math.log(scaling["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo = max(math.floor(dim_of(scaling["fast"])), 0)
    hi = min(math.ceil(dim_of(scaling["slow"])), dims - 1)
    ramp = ((torch.arange(len(inv), dtype=torch.float64) - lo) / max(hi - lo, 0.001)).clamp(0, 1)
    return inv / factor * ramp + inv * (1 - ramp), 0.1 * math.log(factor) + 1.0


def rotary_pairs(dims: int, positions: int, base: float, scaling: Optional[Dict[str, Any]] = None) -> Tensor:
    """float32 ``[positions, dims / 2, 2]``: cosine and sine of ``p * base^(-2i / dims)``, angles in float64; ``scaling``: see
    ``yarn``."""
    inv = base ** (-torch.arange(0, dims, 2, dtype=torch.float64) / max(dims, 1))
    grow = 1.0
    if scaling and dims:
        inv, grow = yarn(inv, base, scaling)
    ang = torch.outer(torch.arange(positions, dtype=torch.float64), inv)
    return (grow * torch.stack((ang.cos(), ang.sin()), dim=-1)).float().contiguous()


class FusedRows(nn.Module):
    """Several matrices ``[rows, in_dim]`` over one input as one matrix.  Every part starts at a multiple of 8 rows
    (zero rows between), so that its columns of the product are 16-byte aligned."""

    def __init__(self, in_dim: int, parts: Sequence[Tuple[str, int, bool]], dtype, device=None):
        super().__init__()
        self.first: Dict[str, int] = {}
        self.rows: Dict[str, int] = {}
        self.biased = [n for n, _, b in parts if b]
        at = 0
        for name, rows, _ in parts:
            self.first[name], self.rows[name] = at, rows
            at += _round8(rows)
        self.weight = _param(at, in_dim, dtype=dtype, device=device)
        self.bias = _param(at, device=device) if self.biased else None
        self._bias_low: Optional[Tensor] = None

    def tensors(self) -> Dict[str, Tensor]:
        out = {}
        for name, at in self.first.items():
            out[name] = self.weight[at:at + self.rows[name]]
            if name in self.biased:
                out[name + ".b"] = self.bias[at:at + self.rows[name]]
        return out

    def forward(self, h: Tensor) -> Tensor:
        if self.bias is None:
            return F.linear(h, self.weight)
        if self._bias_low is None or self._bias_low.dtype != h.dtype or self._bias_low.device != h.device:
            self._bias_low = self.bias.to(h.dtype)
        return F.linear(h, self.weight, self._bias_low)


class Mamba2Mixer(nn.Module):
    """State-space duality (Dao and Gu, "Transformers are SSDs"): one decay per head and token, gate before the norm."""

    def __init__(self, c: Dict[str, Any], eps: float, dtype, device=None):
        super().__init__()
        self.H, self.P, self.N, self.G = c["heads"], c["vdim"], c["state"], c["groups"]
        self.taps, self.norm_groups, self.eps = c["conv"], c["norm_groups"], eps
        self.out_dim = self.H * self.P
        if self.H % self.G or self.out_dim % self.norm_groups:
            raise ValueError("heads must divide into groups and the inner width into norm groups")
        self.channels = self.out_dim + 2 * self.G * self.N
        f = lambda *s: _param(*s, device=device)
        self.conv, self.conv_b = f(self.channels, self.taps), f(self.channels)
        self.dt_bias, self.a_log, self.skip, self.norm = f(self.H), f(self.H), f(self.H), f(self.out_dim)

    def in_parts(self) -> List[Tuple[str, int, bool]]:
        return [("in", self.out_dim + self.channels + self.H, False)]

    def tensors(self) -> Dict[str, Tensor]:
        return {"conv": self.conv, "conv.b": self.conv_b, "dt_bias": self.dt_bias, "A_log": self.a_log, "D": self.skip,
                "norm": self.norm}

    def new_state(self, n_slots: int, n_pages: int, page: int, capacity: int, dtype, device) -> Dict[str, Any]:
        return {"ring": torch.zeros((n_slots, self.taps, self.channels), dtype=dtype, device=device),
                "S": torch.zeros((n_slots, self.H, self.P, self.N), dtype=torch.float32, device=device)}

    def step_sizes_ok(self, rows: int) -> bool:
        return max(self.N, self.P) <= seq_ops.STEP_MAX

    def _columns(self, at: Dict[str, int]) -> Tuple[int, int, int]:
        z = at["in"]
        return z, z + self.out_dim, z + self.out_dim + self.channels

    def prompt(self, proj: Tensor, at: Dict[str, int], b: Batch, st: Dict[str, Any], out: Tensor, scale: float) -> None:
        z, xbc, dt = self._columns(at)
        if b.S >= seq_ops.CHUNKED_MIN and seq_ops.chunked_ok(self.N, self.taps):
            y = seq_ops.ssd_chunked(proj, xbc, dt, self.conv, self.conv_b, st["ring"], self.dt_bias, self.a_log, self.skip, st["S"],
                                    self.H, self.G, self.N, self.P, b)
        else:
            act = seq_ops.conv_silu(proj, xbc, self.conv, self.conv_b, st["ring"], b)
            y = seq_ops.ssd_scan(act, proj, dt, self.dt_bias, self.a_log, self.skip, st["S"], self.H, self.G, self.N, self.P, b)
        seq_ops.conv_push(proj, xbc, self.channels, self.taps, st["ring"], b)
        seq_ops.gated_group_norm(y, proj, z, self._gain(scale), self.eps, self.norm_groups, out)

    def step(self, proj: Tensor, at: Dict[str, int], b: Batch, st: Dict[str, Any], out: Tensor, scale: float) -> None:
        seq_ops.gated_group_norm(self.step_core(proj, at, b, st), proj, self._columns(at)[0], self._gain(scale), self.eps,
                                 self.norm_groups, out)

    def step_core(self, proj: Tensor, at: Dict[str, int], b: Batch, st: Dict[str, Any]) -> Tensor:
        """The step up to its gated norm, which the output projection can take over."""
        _, xbc, dt = self._columns(at)
        return seq_ops.ssd_step(proj, xbc, dt, self.conv, self.conv_b, st["ring"], self.dt_bias, self.a_log, self.skip, st["S"],
                                self.H, self.G, self.N, self.P, b)

    def _gain(self, scale: float) -> Tensor:
        return self.norm if scale == 1.0 else self.norm * scale


class ChannelDeltaMixer(nn.Module):
    """Gated delta rule with a decay per head and key channel, low-rank decay and output-gate projections."""

    def __init__(self, c: Dict[str, Any], eps: float, ranks: Tuple[int, int], dtype, device=None):
        super().__init__()
        self.H, self.G, self.D, self.E, self.taps, self.eps = c["heads"], c["kv_heads"], c["dim"], c["vdim"], c["conv"], eps
        if self.H % self.G:
            raise ValueError("heads must divide into kv heads")
        self.rank_a, self.rank_g = ranks
        self.out_dim = self.H * self.E
        self.split = (self.G * self.D, self.G * self.D, self.H * self.E)
        f = lambda *s: _param(*s, device=device)
        self.conv = f(sum(self.split), self.taps)
        self.a_log, self.dt_bias, self.norm = f(self.H), f(self.H * self.D), f(self.E)
        # second factors, their ranks padded with zeros to whole 16-byte pieces
        self.a2 = _param(self.H * self.D, _round8(self.rank_a), dtype=dtype, device=device)
        self.g2 = _param(self.H * self.E, _round8(self.rank_g), dtype=dtype, device=device)

    def in_parts(self) -> List[Tuple[str, int, bool]]:
        q, k, v = self.split
        # q | k | v are convolved together and have to touch; the low ranks read as whole pieces
        return [("qkv", q + k + v, False), ("b", self.H, False), ("a1", self.rank_a, False), ("g1", self.rank_g, False)]

    def step_sizes_ok(self, rows: int) -> bool:
        return max(self.D, self.E) <= seq_ops.STEP_MAX

    def sub_parts(self) -> Dict[str, Tuple[str, int, int]]:
        """Checkpoint tensors that are slices of one part: name -> (part, first row, rows)."""
        q, k, v = self.split
        return {"q": ("qkv", 0, q), "k": ("qkv", q, k), "v": ("qkv", q + k, v)}

    def tensors(self) -> Dict[str, Tensor]:
        q, k, v = self.split
        return {"q.conv": self.conv[:q], "k.conv": self.conv[q:q + k], "v.conv": self.conv[q + k:], "A_log": self.a_log,
                "dt_bias": self.dt_bias, "norm": self.norm, "a2": self.a2[:, :self.rank_a], "g2": self.g2[:, :self.rank_g]}

    def new_state(self, n_slots: int, n_pages: int, page: int, capacity: int, dtype, device) -> Dict[str, Any]:
        return {"ring": torch.zeros((n_slots, self.taps, sum(self.split)), dtype=dtype, device=device),
                "S": torch.zeros((n_slots, self.H, self.E, self.D), dtype=torch.float32, device=device)}

    def prompt(self, proj: Tensor, at: Dict[str, int], b: Batch, st: Dict[str, Any], out: Tensor, scale: float) -> None:
        qkv, a1, g1 = at["qkv"], at["a1"], at["g1"]
        raw = F.linear(proj[:, a1:a1 + self.a2.shape[1]], self.a2)
        gate = F.linear(proj[:, g1:g1 + self.g2.shape[1]], self.g2)
        args = (proj, qkv, raw, at["b"], self.conv, st["ring"], self.a_log, self.dt_bias)
        if b.S >= seq_ops.CHUNKED_MIN and seq_ops.chunked_ok(self.D, self.taps):
            o = seq_ops.delta_chunked(*args, st["S"], self.H, self.G, self.D, self.E, b)
        else:
            q, k, v, decay, beta = seq_ops.delta_prep(*args, self.H, self.G, self.D, self.E, b)
            o = seq_ops.delta_scan(q, k, v, decay, beta, st["S"], b)
        seq_ops.conv_push(proj, qkv, sum(self.split), self.taps, st["ring"], b)
        seq_ops.head_norm_gate(o, gate, self.norm, self.eps, scale, out)

    def step(self, proj: Tensor, at: Dict[str, int], b: Batch, st: Dict[str, Any], out: Tensor, scale: float) -> None:
        seq_ops.delta_step(proj, at["qkv"], at["b"], at["a1"], at["g1"], self.conv, st["ring"], self.a2, self.g2, self.a_log,
                           self.dt_bias, self.norm, self.eps, scale, st["S"], out, self.H, self.G, self.D, self.E, b)


class WindowAttention(nn.Module):
    """Grouped-query attention over the last ``mask.size`` positions, head norms in front of the rotation, one
    sigmoid gate per head behind; keys and values may differ in size."""

    def __init__(self, c: Dict[str, Any], eps: float, dtype, device=None):
        super().__init__()
        self.spec = WindowAttnSpec(c["heads"], c["kv_heads"], c["dim"], c["vdim"], int(c["mask"]["size"]), float(c["scale"]),
                                   int(c["rot"]["dims"]), eps)
        s = self.spec
        if s.H % s.G or s.rot % 2 or s.rot > s.D or s.window < 1:
            raise ValueError("bad attention sizes: heads over kv heads, an even number of rotated dimensions, a window of 1 or more")
        self.base = float(c["rot"]["base"])
        self.out_dim = s.H * s.E
        self.q_norm, self.k_norm = _param(s.D, device=device), _param(s.D, device=device)

    def step_sizes_ok(self, rows: int) -> bool:
        return True

    def in_parts(self) -> List[Tuple[str, int, bool]]:
        s = self.spec
        return [("q", s.H * s.D, True), ("k", s.G * s.D, True), ("v", s.G * s.E, True), ("g", s.H, False)]

    def tensors(self) -> Dict[str, Tensor]:
        return {"q.norm": self.q_norm, "k.norm": self.k_norm}

    def new_state(self, n_slots: int, n_pages: int, page: int, capacity: int, dtype, device) -> Dict[str, Any]:
        s = self.spec
        kv = PagedKV(n_pages, page, s.G, s.D, device, dtype, v_head_dim=s.E)
        return {"kv": kv, "cs": rotary_pairs(s.rot, capacity, self.base).to(device)}

    def prompt(self, proj: Tensor, at: Dict[str, int], b: Batch, st: Dict[str, Any], out: Tensor, scale: float,
               simple: bool = False) -> None:
        kv = st["kv"]
        q = seq_ops.attn_prep(proj, at["q"], at["k"], at["v"], self.q_norm, self.k_norm, st["cs"], kv.k, kv.v, self.spec, b)
        seq_ops.attn_window(q, kv.k, kv.v, proj, at["g"], scale, self.spec, b, out, simple)

    def step(self, proj: Tensor, at: Dict[str, int], b: Batch, st: Dict[str, Any], out: Tensor, scale: float) -> None:
        kv = st["kv"]
        if not seq_ops.attn_decode_ok(self.spec, kv.page_size):
            return self.prompt(proj, at, b, st, out, scale, simple=True)
        seq_ops.attn_decode(proj, at["q"], at["k"], at["v"], at["g"], self.q_norm, self.k_norm, st["cs"], kv.k, kv.v, scale,
                            self.spec, b, out)


class LatentAttention(nn.Module):
    """Attention whose queries, keys and values pass through low-rank latents (Multi-head Latent Attention of DeepSeek-AI,
    "DeepSeek-V2"), over the last ``mask.size`` positions, gated element by element.  A position caches its normed latent and
    one rotated key part that all heads share.  Prompts form keys and values of all heads by one product over the cached
    rows that their windows reach; single tokens move the two factors to the query and to the output."""

    def __init__(self, c: Dict[str, Any], eps: float, dtype, device=None):
        super().__init__()
        rot = c["rot"]
        self.spec = s = LatentSpec(c["heads"], c["dim"], c["rot_dim"], int(rot["dims"]), c["vdim"], c["q_rank"], c["kv_rank"],
                                   int(c["mask"]["size"]), float(c["scale"]), eps)
        if s.rd % 2 or s.rd > s.rot or s.window < 1:
            raise ValueError("bad attention sizes: an even number of rotated dimensions among rot_dim, a window of 1 or more")
        self.base, self.scaling = float(rot["base"]), rot.get("scaling")
        self.out_dim, self.window = s.H * s.E, s.window
        self.q_norm, self.kv_norm = _param(s.QR, device=device), _param(s.R, device=device)
        self.uq = _param(s.H * (s.dim + s.rot), s.QR, dtype=dtype, device=device)
        self.ukv = _param(s.H * (s.dim + s.E), s.R, dtype=dtype, device=device)  # key factors of all heads, then value factors

    def step_sizes_ok(self, rows: int, page: int = 64) -> bool:
        return seq_ops.gemv_ok(rows, self.uq) and seq_ops.latent_decode_ok(self.spec, rows, page)

    def in_parts(self) -> List[Tuple[str, int, bool]]:
        s = self.spec
        return [("dq", s.QR, False), ("dkv", s.R + s.rot, False), ("g", s.H * s.E, False)]

    def tensors(self) -> Dict[str, Tensor]:
        keys = self.spec.H * self.spec.dim
        return {"dq.norm": self.q_norm, "dkv.norm": self.kv_norm, "uq": self.uq, "uk": self.ukv[:keys], "uv": self.ukv[keys:]}

    def new_state(self, n_slots: int, n_pages: int, page: int, capacity: int, dtype, device) -> Dict[str, Any]:
        s = self.spec
        return {"kv": PagedKV(n_pages, page, 1, s.R + s.rot, device, dtype, v_head_dim=0),
                "cs": rotary_pairs(s.rd, capacity, self.base, self.scaling).to(device)}

    def prompt(self, proj: Tensor, at: Dict[str, int], b: Batch, st: Dict[str, Any], out: Tensor, scale: float,
               simple: bool = False) -> None:
        s, kc = self.spec, st["kv"].k
        cq, packed = seq_ops.latent_prep(proj, at["dq"], at["dkv"], self.q_norm, self.kv_norm, st["cs"], kc, s, b)
        q = F.linear(cq, self.uq)
        seq_ops.latent_rotate(q, st["cs"], s, b)
        seq_ops.latent_window(q, F.linear(packed[:, :s.R], self.ukv), packed, proj, at["g"], s, b, out, simple)
        if scale != 1.0:
            out.mul_(scale)

    def step(self, proj: Tensor, at: Dict[str, int], b: Batch, st: Dict[str, Any], out: Tensor, scale: float) -> None:
        s, kv = self.spec, st["kv"]
        if scale != 1.0 or not seq_ops.latent_decode_ok(s, b.B, kv.page_size):
            return self.prompt(proj, at, b, st, out, scale, simple=True)
        q = seq_ops.row_norm_gemv(proj, at["dq"], self.q_norm, s.eps, self.uq)
        keys = s.H * s.dim
        seq_ops.latent_decode(proj, at["dkv"], at["g"], q, self.ukv[:keys], self.ukv[keys:], self.kv_norm, st["cs"], kv.k, s, b, out)


class LightningMixer(nn.Module):
    """Linear attention with a constant decay per head (Lightning Attention): ``S <- decay S + k v^T, o = S^T q`` of SiLU'd
    projections, all heads normed together, gated element by element.  It runs on the state-space kernels: v, k and q are
    their x, B and C of as many groups as heads, behind a convolution of one tap with weight 1 (so only its SiLU is left),
    with step size 1."""

    def __init__(self, c: Dict[str, Any], eps: float, dtype, device=None):
        super().__init__()
        self.H, self.D, self.E, self.eps = c["heads"], c["dim"], c["vdim"], eps
        if len(c["decay"]) != self.H or not all(0 < d <= 1 for d in c["decay"]):
            raise ValueError("one decay per head is needed, above 0 and at most 1")
        self.out_dim, self.channels = self.H * self.E, self.H * (self.E + 2 * self.D)
        self.norm = _param(self.out_dim, device=device)
        for name, t in (("decay", torch.tensor([float(d) for d in c["decay"]], dtype=torch.float32)),
                        ("tap", torch.ones(self.channels, 1)), ("tap_b", torch.zeros(self.channels))):
            self.register_buffer(name, t.to(device), persistent=False)

    def in_parts(self) -> List[Tuple[str, int, bool]]:
        return [("vkq", self.channels, False), ("g", self.out_dim, False)]

    def sub_parts(self) -> Dict[str, Tuple[str, int, int]]:
        v, k = self.out_dim, self.H * self.D
        return {"v": ("vkq", 0, v), "k": ("vkq", v, k), "q": ("vkq", v + k, k)}

    def tensors(self) -> Dict[str, Tensor]:
        return {"norm": self.norm}

    def step_sizes_ok(self, rows: int) -> bool:
        return max(self.D, self.E) <= seq_ops.STEP_MAX and self.out_dim % 8 == 0

    def new_state(self, n_slots: int, n_pages: int, page: int, capacity: int, dtype, device) -> Dict[str, Any]:
        return {"ring": torch.zeros((n_slots, 1, self.channels), dtype=dtype, device=device),
                "S": torch.zeros((n_slots, self.H, self.E, self.D), dtype=torch.float32, device=device)}

    def _args(self, st):
        return None, None, None, st["S"], self.H, self.H, self.D, self.E

    def prompt(self, proj: Tensor, at: Dict[str, int], b: Batch, st: Dict[str, Any], out: Tensor, scale: float) -> None:
        if b.S >= seq_ops.CHUNKED_MIN and seq_ops.chunked_ok(self.D, 1):
            y = seq_ops.ssd_chunked(proj, at["vkq"], 0, self.tap, self.tap_b, st["ring"], *self._args(st), b, self.decay)
        else:
            act = seq_ops.conv_silu(proj, at["vkq"], self.tap, self.tap_b, st["ring"], b)
            y = seq_ops.ssd_scan(act, proj, 0, *self._args(st), b, self.decay)
        seq_ops.norm_gate(y, proj, at["g"], self._gain(scale), self.eps, out)

    def step_core(self, proj: Tensor, at: Dict[str, int], b: Batch, st: Dict[str, Any]) -> Tensor:
        return seq_ops.ssd_step(proj, at["vkq"], 0, self.tap, self.tap_b, st["ring"], *self._args(st), b, self.decay)

    def step(self, proj: Tensor, at: Dict[str, int], b: Batch, st: Dict[str, Any], out: Tensor, scale: float) -> None:
        seq_ops.norm_gate(self.step_core(proj, at, b, st), proj, at["g"], self._gain(scale), self.eps, out)

    def step_out(self, proj: Tensor, at: Dict[str, int], b: Batch, st: Dict[str, Any], w: Tensor) -> Tensor:
        """The step with norm, gate and the output projection ``w`` (fp32) in one launch behind the recurrence."""
        return seq_ops.norm_gate_gemv_f32(self.step_core(proj, at, b, st), proj, at["g"], self.norm, self.eps, w)

    def _gain(self, scale: float) -> Tensor:
        return self.norm if scale == 1.0 else self.norm * scale


class MixerBlock(nn.Module):
    """One mixer, or several side by side on the same input: ``sum_i scale_i * W_o_i mixer_i(W_in_i h)`` with one
    product in front and one behind (the scales are applied to the mixers' outputs, in fp32)."""

    def __init__(self, width: int, mixers: Sequence[Tuple[str, nn.Module, float]], dtype, device=None):
        super().__init__()
        self.prefixes = [p for p, _, _ in mixers]
        self.scales = [float(s) for _, _, s in mixers]
        self.mixers = nn.ModuleList([m for _, m, _ in mixers])
        parts = [(p + n, rows, bias) for p, m, _ in mixers for n, rows, bias in m.in_parts()]
        self.w_in = FusedRows(width, parts, dtype, device)
        self.inner = sum(m.out_dim for m in self.mixers)
        self.w_out = _param(width, self.inner, dtype=dtype, device=device)
        # first column of every part of the product, by the names the mixer uses
        self.at = [{n: self.w_in.first[p + n] for n, _, _ in m.in_parts()} for p, m, _ in mixers]

    def tensors(self) -> Dict[str, Tensor]:
        rows, out, col = self.w_in.tensors(), {}, 0
        for p, m in zip(self.prefixes, self.mixers):
            sub = m.sub_parts() if hasattr(m, "sub_parts") else {}
            split = {part for part, _, _ in sub.values()}
            for name, _, bias in m.in_parts():
                for n in ([name] if name not in split else []) + ([name + ".b"] if bias else []):
                    out[p + n] = rows[p + n]
            for name, (part, first, n) in sub.items():
                out[p + name] = rows[p + part][first:first + n]
            out.update({p + n: t for n, t in m.tensors().items()})
            out[p + "o"] = self.w_out[:, col:col + m.out_dim]
            col += m.out_dim
        return out

    def new_state(self, *args) -> List[Dict[str, Any]]:
        return [m.new_state(*args) for m in self.mixers]

    def _run(self, proj: Tensor, b: Batch, st, form: str) -> Tensor:
        out = torch.empty((proj.shape[0], self.inner), dtype=proj.dtype, device=proj.device)
        col = 0
        for m, at, scale, s in zip(self.mixers, self.at, self.scales, st):
            getattr(m, form)(proj, at, b, s, out[:, col:col + m.out_dim], scale)
            col += m.out_dim
        return out

    def prompt(self, h: Tensor, b: Batch, st) -> Branch:
        return Branch(F.linear(self._run(self.w_in(h), b, st, "prompt"), self.w_out))

    def step(self, s: Stream, gain: Tensor, b: Batch, st, post: Optional[Tensor]) -> None:
        """``x += mult * mixer(norm(x))`` for one token per sequence; with ``post``, the output is left pending."""
        proj = s.norm_gemv(gain, self.w_in.weight, self.w_in.bias)
        m, alone = self.mixers[0], len(self.mixers) == 1 and self.scales[0] == 1.0
        if post is not None:
            s.y = m.step_out(proj, self.at[0], b, st[0], self.w_out) if alone and hasattr(m, "step_out") \
                else seq_ops.gemv_f32(self._run(proj, b, st, "step"), self.w_out)
            s.post = post
        elif alone and isinstance(m, Mamba2Mixer):
            y = m.step_core(proj, self.at[0], b, st[0])
            seq_ops.gated_norm_gemv_residual(y, proj, m._columns(self.at[0])[0], m.norm, m.eps, m.norm_groups, self.w_out, s.mult, s.x)
        else:
            seq_ops.gemv_residual(self._run(proj, b, st, "step"), self.w_out, s.mult, s.x)

    def step_ok(self, rows: int) -> bool:
        return seq_ops.gemv_ok(rows, self.w_in.weight) and seq_ops.gemv_ok(rows, self.w_out) \
            and all(m.step_sizes_ok(rows) for m in self.mixers)


class ClampedGLU(nn.Module):
    """``W_down (g sigmoid(1.702 g) (u + 1))`` with ``g = min(W_gate h, limit)`` and ``u`` clamped to ``+- limit``."""

    def __init__(self, width: int, c: Dict[str, Any], dtype, device=None):
        super().__init__()
        self.ff, self.limit = int(c["ff"]), float(c["limit"])
        self.gate_up = _param(2 * self.ff, width, dtype=dtype, device=device)
        self.down = _param(width, self.ff, dtype=dtype, device=device)

    def tensors(self) -> Dict[str, Tensor]:
        return {"gate": self.gate_up[:self.ff], "up": self.gate_up[self.ff:], "down": self.down}

    def prompt(self, h: Tensor) -> Branch:
        return Branch(F.linear(seq_ops.clamped_glu(F.linear(h, self.gate_up), self.limit), self.down))

    def step(self, s: Stream, gain: Tensor, post: Optional[Tensor]) -> None:
        act = s.norm_gemv_glu(gain, self.gate_up, self.limit)
        if post is None:
            seq_ops.gemv_residual(act, self.down, s.mult, s.x)
        else:
            s.y, s.post = seq_ops.gemv_f32(act, self.down), post

    def step_ok(self, rows: int) -> bool:
        return seq_ops.gemv_ok(rows, self.gate_up) and seq_ops.gemv_ok(rows, self.down)


class RoutedExperts(nn.Module):
    """``sum_e W_down_e glu(W_gate_e (s_e h), W_up_e (s_e h))`` over the ``top`` experts with the largest scores
    ``s = sigmoid(W_router h)`` (not renormalised; the score scales the expert's input), ``glu(g, u) = silu(g) u``; plus a
    shared expert that every token passes."""

    def __init__(self, width: int, c: Dict[str, Any], dtype, device=None):
        super().__init__()
        self.Ex, self.top, self.ff = int(c["router"]["experts"]), int(c["router"]["top"]), int(c["expert"]["ff"])
        self.shared_ff = int(c["shared"]["ff"]) if c.get("shared") else 0
        if not 0 < self.top <= self.Ex:
            raise ValueError("a token's experts must be at least one and at most all of them")
        # one matrix that reads the normed stream: the router's rows, then the shared expert's gate and up rows
        self.front = _param(self.Ex + 2 * self.shared_ff, width, dtype=dtype, device=device)
        self.gate_up = _param(self.Ex, 2 * self.ff, width, dtype=dtype, device=device)
        self.down = _param(self.Ex, width, self.ff, dtype=dtype, device=device)
        self.shared_down = _param(width, self.shared_ff, dtype=dtype, device=device) if self.shared_ff else None

    def tensors(self) -> Dict[str, Tensor]:
        out = {"router": self.front[:self.Ex]}
        for e in range(self.Ex):
            out.update({f"e{e}.gate": self.gate_up[e, :self.ff], f"e{e}.up": self.gate_up[e, self.ff:], f"e{e}.down": self.down[e]})
        if self.shared_ff:
            gate = self.Ex + self.shared_ff
            out.update({"shared.gate": self.front[self.Ex:gate], "shared.up": self.front[gate:], "shared.down": self.shared_down})
        return out

    def prompt(self, h: Tensor) -> Branch:
        ids, scores = seq_ops.moe_route(h, self.front[:self.Ex], self.top)
        y = F.linear(seq_ops.silu_glu(F.linear(h, self.front[self.Ex:])), self.shared_down) if self.shared_ff else None
        return Branch(y, seq_ops.moe_experts(h, ids, scores, self.gate_up, self.down))

    def step(self, s: Stream, gain: Tensor, post: Optional[Tensor]) -> None:
        z, shared, h = s.norm_route(gain, self.front, self.Ex)
        y = seq_ops.moe_step(h, z, self.top, self.gate_up, self.down, *((shared, self.shared_down) if self.shared_ff else ()))
        s.y, s.post = y, post

    def step_ok(self, rows: int) -> bool:
        return self.shared_ff > 0 and seq_ops.gemv_ok(rows, self.front) \
            and seq_ops.moe_step_ok(rows, self.front.shape[1], self.ff, self.shared_ff, self.Ex, self.top)
