"""Token mixers of the hybrid decoders beside ``block.GQA``: sliding-window attention, the gated delta rule
with one decay per key channel, the Mamba-2 state-space mixer, and their composition side by side.

A mixer reads columns of one fused input projection and writes columns of the input of one fused output
projection; ``MixerBlock`` owns both matrices.  So mixers that read the same input side by side cost one
product in front and one behind, whatever they are.  Each mixer has two forms: ``prompt`` for any number of
new tokens per sequence (convolution, scan, norm as separate launches around the vendor's matrix products)
and ``step`` for one new token per sequence (everything between the two projections in one launch).

Weights are kept under the names their checkpoint uses; ``tensors()`` of every module maps those names to
(views of) its parameters.
"""
from __future__ import annotations

from typing import Any, Dict, List, Optional, Sequence, Tuple

import torch
import torch.nn as nn
import torch.nn.functional as F
from torch import Tensor

from . import seq_ops
from .block import PagedKV
from .seq_ops import Batch, WindowAttnSpec


def _round8(n: int) -> int:
    return (n + 7) // 8 * 8


def _param(*shape, dtype=torch.float32, device=None) -> nn.Parameter:
    return nn.Parameter(torch.zeros(shape, dtype=dtype, device=device), requires_grad=False)


def rotary_pairs(dims: int, positions: int, base: float) -> Tensor:
    """float32 ``[positions, dims / 2, 2]``: cosine and sine of ``p * base^(-2i / dims)``, angles in float64."""
    inv = base ** (-torch.arange(0, dims, 2, dtype=torch.float64) / max(dims, 1))
    ang = torch.outer(torch.arange(positions, dtype=torch.float64), inv)
    return torch.stack((ang.cos(), ang.sin()), dim=-1).float().contiguous()


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

    def step_sizes_ok(self) -> bool:
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

    def step_sizes_ok(self) -> bool:
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

    def step_sizes_ok(self) -> bool:
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

    def prompt(self, h: Tensor, b: Batch, st) -> Tensor:
        return F.linear(self._run(self.w_in(h), b, st, "prompt"), self.w_out)

    def step(self, x: Tensor, gain: Tensor, eps: float, b: Batch, st, mult: float) -> None:
        """``x += mult * mixer(norm(x))`` for one token per sequence."""
        proj = seq_ops.norm_gemv(x, gain, eps, self.w_in.weight, self.w_in.bias)
        m = self.mixers[0]
        if len(self.mixers) == 1 and hasattr(m, "step_core") and self.scales[0] == 1.0:
            y = m.step_core(proj, self.at[0], b, st[0])
            seq_ops.gated_norm_gemv_residual(y, proj, m._columns(self.at[0])[0], m.norm, m.eps, m.norm_groups, self.w_out, mult, x)
        else:
            seq_ops.gemv_residual(self._run(proj, b, st, "step"), self.w_out, mult, x)

    def step_ok(self, rows: int) -> bool:
        return seq_ops.gemv_ok(rows, self.w_in.weight) and seq_ops.gemv_ok(rows, self.w_out) \
            and all(m.step_sizes_ok() for m in self.mixers)


class ClampedGLU(nn.Module):
    """``W_down (g sigmoid(1.702 g) (u + 1))`` with ``g = min(W_gate h, limit)`` and ``u`` clamped to ``+- limit``."""

    def __init__(self, width: int, c: Dict[str, Any], dtype, device=None):
        super().__init__()
        self.ff, self.limit = int(c["ff"]), float(c["limit"])
        self.gate_up = _param(2 * self.ff, width, dtype=dtype, device=device)
        self.down = _param(width, self.ff, dtype=dtype, device=device)

    def tensors(self) -> Dict[str, Tensor]:
        return {"gate": self.gate_up[:self.ff], "up": self.gate_up[self.ff:], "down": self.down}

    def prompt(self, h: Tensor) -> Tensor:
        return F.linear(seq_ops.clamped_glu(F.linear(h, self.gate_up), self.limit), self.down)

    def step(self, x: Tensor, gain: Tensor, eps: float, mult: float) -> None:
        seq_ops.gemv_residual(seq_ops.norm_gemv_glu(x, gain, eps, self.gate_up, self.limit), self.down, mult, x)

    def step_ok(self, rows: int) -> bool:
        return seq_ops.gemv_ok(rows, self.gate_up) and seq_ops.gemv_ok(rows, self.down)
