"""Tensor-level operators over libastrai_seq.so (include/astrai_seq.h): the row operations, matrix-vector
products, convolutions, linear recurrences, windowed and latent attention and routed experts of the hybrid decoders.

As in ``ops``: tensors already on the GPU, layouts checked as the kernels assume them, work queued on
torch's current stream, no CPU fallback.  ``proj`` arguments are rows of a fused projection
``[M, ld]``; ``o_*`` are first columns of its parts.
"""
from __future__ import annotations

from typing import NamedTuple, Optional, Tuple

import torch
from torch import Tensor

from . import _abi
from .ops import _DT, _need_gpu, _OnDevice, _stream


class Batch(NamedTuple):
    """The sequences of one step: ``S`` new tokens each, from position ``pos[b]`` on.  ``pos`` and ``slots`` int32
    ``[B]``, ``table`` int64 ``[B, P]`` (physical pages of each sequence, -1 where none), all on the device.  ``starts``:
    the positions as the host knows them, or None (a captured step)."""
    pos: Tensor
    slots: Tensor
    table: Tensor
    B: int
    S: int
    starts: Optional[Tuple[int, ...]] = None


def _call(name: str, dev: torch.device, *args) -> None:
    with _OnDevice(dev):
        rc = getattr(_abi.load_seq(), name)(*args)
    _abi.check(rc, name)


def _p(t: Optional[Tensor], col: int = 0):
    return None if t is None else t.data_ptr() + col * t.element_size()


def _rows2(t: Tensor, what: str, dtype=None) -> Tensor:
    if t.dim() != 2 or (t.shape[0] > 1 and t.stride(1) != 1) or (dtype is not None and t.dtype != dtype):
        raise ValueError(f"{what} must be rows [M, K] with contiguous columns, got {tuple(t.shape)} {t.dtype}")
    return t


def _vec(t: Optional[Tensor], n: int, what: str) -> None:
    if t is not None and (t.dtype != torch.float32 or t.numel() != n or not t.is_contiguous()):
        raise ValueError(f"{what} must be {n} contiguous float32 elements, got {t.dtype} {tuple(t.shape)}")


def _batch(b: Batch, rows: int, n_slots: Optional[int] = None) -> None:
    if b.pos.dtype != torch.int32 or b.slots.dtype != torch.int32 or b.pos.numel() != b.B or b.slots.numel() != b.B:
        raise ValueError("pos and slots must be int32 [B]")
    if b.table.dtype != torch.int64 or b.table.dim() != 2 or b.table.shape[0] != b.B or not b.table.is_contiguous():
        raise ValueError("table must be contiguous int64 [B, P]")
    if rows != b.B * b.S:
        raise ValueError(f"{rows} rows for {b.B} sequences of {b.S} tokens")


# ------------------------------------------------------------------------------------------------ rows
def embed(ids: Tensor, table: Tensor) -> Tensor:
    """fp32 rows of ``table [V, K]``; an id outside the table is a zero row."""
    _need_gpu(ids, table)
    if ids.dtype != torch.int64 or table.dim() != 2 or not table.is_contiguous():
        raise ValueError("ids must be int64 and the table contiguous [V, K]")
    ids = ids.reshape(-1).contiguous()
    x = torch.empty((ids.numel(), table.shape[1]), dtype=torch.float32, device=table.device)
    _call("aqs_embed", x.device, _p(ids), _p(table), _DT[table.dtype], _p(x), x.shape[0], x.shape[1], table.shape[0], _stream(x))
    return x


class Routed(NamedTuple):
    """Rows ``[A, K]`` of chosen experts; token m's are ``slots[m]`` (int32 ``[M, top]``)."""
    rows: Tensor
    slots: Tensor


def add_rmsnorm(x: Tensor, y: Optional[Tensor], mult: float, w: Optional[Tensor], eps: float, dtype: torch.dtype,
                norm: bool = True, w0: float = 1.0, post: Optional[Tensor] = None, routed: Optional[Routed] = None) -> Optional[Tensor]:
    """``x += mult * t`` in place (fp32 ``x [M, K]``), then ``rms(x) * (w0 + w)`` as ``dtype``.  The branch output t is
    ``y`` (optional) plus each token's ``routed`` rows, normed with weight ``post`` if that is given."""
    _need_gpu(x, y, w, post)
    M, K = x.shape
    if x.dtype != torch.float32 or not x.is_contiguous() or (y is not None and (y.shape != x.shape or y.dtype != dtype)):
        raise ValueError("x must be contiguous float32 [M, K] and y have its shape")
    if y is not None:
        _rows2(y, "y")
    _vec(w, K, "w")
    _vec(post, K, "post")
    top = 0
    if routed is not None:
        top = routed.slots.shape[1]
        if routed.rows.dtype != dtype or routed.rows.shape[1:] != (K,) or not routed.rows.is_contiguous() \
                or routed.slots.dtype != torch.int32 or routed.slots.shape[0] != M or not routed.slots.is_contiguous():
            raise ValueError(f"routed rows must be contiguous {dtype} [A, {K}] with int32 slots [{M}, top]")
    branch = y is not None or top > 0
    out = torch.empty((M, K), dtype=dtype, device=x.device) if norm else None
    if M and (norm or branch):
        _call("aqs_add_rmsnorm", x.device, _p(x), _p(y), y.stride(0) if y is not None else K, _DT[dtype],
              _p(routed.rows) if top else None, _p(routed.slots) if top else None, top, _p(post) if branch else None, float(mult), _p(w),
              float(w0), float(eps), _p(out), M, K, _stream(x))
    return out


def silu_glu(gu: Tensor) -> Tensor:
    """``gu [M, 2F] = gate | up`` -> ``silu(gate) * up``."""
    _need_gpu(gu)
    _rows2(gu, "gu")
    M, F = gu.shape[0], gu.shape[1] // 2
    out = torch.empty((M, F), dtype=gu.dtype, device=gu.device)
    _call("aqs_silu_glu", gu.device, _p(gu), gu.stride(0), _DT[gu.dtype], _p(out), M, F, _stream(gu))
    return out


def norm_gate(y: Tensor, proj: Tensor, o_z: int, w: Tensor, eps: float, out: Tensor) -> None:
    """``out = rms(y) * w * sigmoid(z)`` (fp32 ``y [M, K]``), z the columns of ``proj`` from ``o_z`` on."""
    _need_gpu(y, proj, w, out)
    M, K = y.shape
    _rows2(out, "out", proj.dtype)
    _vec(w, K, "w")
    if y.dtype != torch.float32 or not y.is_contiguous() or proj.shape[0] != M or o_z + K > proj.shape[1] or out.shape != y.shape:
        raise ValueError("norm_gate: shapes do not fit")
    _call("aqs_norm_gate", y.device, _p(y), _p(proj, o_z), proj.stride(0), _DT[proj.dtype], _p(w), float(eps), _p(out), out.stride(0),
          M, K, _stream(y))


def clamped_glu(gu: Tensor, limit: float) -> Tensor:
    """``gu [M, 2F] = gate | up`` -> ``g sigmoid(1.702 g) (u + 1)`` with g capped and u clamped at ``limit``."""
    _need_gpu(gu)
    _rows2(gu, "gu")
    M, F = gu.shape[0], gu.shape[1] // 2
    out = torch.empty((M, F), dtype=gu.dtype, device=gu.device)
    _call("aqs_clamped_glu", gu.device, _p(gu), gu.stride(0), _DT[gu.dtype], float(limit), _p(out), M, F, _stream(gu))
    return out


def gated_group_norm(y: Tensor, proj: Tensor, o_z: int, w: Tensor, eps: float, groups: int, out: Tensor) -> None:
    """``out = rms(y * silu(z)) * w`` with the RMS over each of ``groups`` equal parts; z the columns of ``proj`` from
    ``o_z`` on."""
    _need_gpu(y, proj, w, out)
    M, K = y.shape
    _rows2(out, "out", proj.dtype)
    _vec(w, K, "w")
    if y.dtype != torch.float32 or not y.is_contiguous() or proj.shape[0] != M or o_z + K > proj.shape[1] or out.shape != y.shape:
        raise ValueError("gated_group_norm: shapes do not fit")
    _call("aqs_gated_group_norm", y.device, _p(y), _p(proj, o_z), proj.stride(0), _DT[proj.dtype], _p(w), float(eps), _p(out),
          out.stride(0), M, K, int(groups), _stream(y))


def head_norm_gate(o: Tensor, gate: Tensor, w: Tensor, eps: float, scale: float, out: Tensor) -> None:
    """Each head of ``o [M, H, E]`` over its root mean square, times ``w [E]``, ``sigmoid(gate [M, H*E])`` and ``scale``."""
    _need_gpu(o, gate, w, out)
    M, H, E = o.shape
    _rows2(out, "out", gate.dtype)
    _vec(w, E, "w")
    if o.dtype != torch.float32 or not o.is_contiguous() or gate.shape != (M, H * E) or out.shape != (M, H * E):
        raise ValueError("head_norm_gate: shapes do not fit")
    _call("aqs_head_norm_gate", o.device, _p(o), _p(gate), gate.stride(0), _DT[gate.dtype], _p(w), float(eps), float(scale),
          _p(out), out.stride(0), M, H, E, _stream(o))


# ------------------------------------------------------------------------------------------------ matrix-vector products
def gemv_ok(M: int, w: Tensor) -> bool:
    """Whether the products with ``w [N, K]`` below serve M rows."""
    return bool(_abi.load_seq().aqs_gemv_ok(_DT[w.dtype], M, w.shape[0], w.shape[1]))


def _gemv(in_kind, out_kind, w, x=None, ldx=0, o_x=0, xf=None, yf=None, post=None, x_out=None, gain=None, gain0=0.0, eps=0.0, groups=1,
          bias=None, mult=0.0, limit=0.0, routers=0, res=None, out=None, h_out=None):
    _need_gpu(w, x, xf, yf, post, x_out, gain, bias, res, out, h_out)
    N, K = w.shape
    if not w.is_contiguous():
        raise ValueError("weights must be contiguous [N, K]")
    if xf is not None and (xf.dtype != torch.float32 or xf.dim() != 2 or xf.shape[1] != K or not xf.is_contiguous()):
        raise ValueError(f"fp32 rows must be contiguous [M, {K}], got {tuple(xf.shape)}")
    for t in (yf, x_out):
        if t is not None and (t.dtype != torch.float32 or t.shape != xf.shape or not t.is_contiguous()):
            raise ValueError("the branch output and the new stream must be like the stream")
    if x is not None and (x.dtype != w.dtype or x.dim() != 2 or o_x + K > x.shape[1]):
        raise ValueError(f"rows must be {w.dtype} [M, {K}], got {x.dtype} {tuple(x.shape)}")
    _vec(gain, K, "gain")
    _vec(post, K, "post")
    _vec(bias, N, "bias")
    M = (xf if xf is not None else x).shape[0]
    dst = out if out is not None else res
    _call("aqs_gemv", w.device, in_kind, out_kind, _DT[w.dtype], _p(x, o_x), ldx, _p(xf), _p(yf), _p(post), _p(x_out), _p(gain),
          float(gain0), float(eps), int(groups), _p(w), _p(bias), float(mult), float(limit), int(routers), _p(res), _p(out), dst.stride(0),
          _p(h_out), M, N, K, _stream(w))


class Stream:
    """The fp32 residual rows ``x [M, K]`` of a one-token step.  A branch output ``y`` whose own norm (weight ``post``) and
    addition are still to come is taken in by the product that reads the stream next."""

    def __init__(self, x: Tensor, eps: float, w0: float, mult: float):
        self.x, self.eps, self.w0, self.mult = x, eps, w0, mult
        self.y: Optional[Tensor] = None
        self.post: Optional[Tensor] = None

    def _front(self, gain):
        """(in_kind, arguments) of a product behind the norm with weight ``w0 + gain``; the pending output is added."""
        args = dict(xf=self.x, gain=gain, gain0=self.w0, eps=self.eps)
        if self.y is None:
            return 1, args
        args.update(yf=self.y, post=self.post, mult=self.mult, x_out=torch.empty_like(self.x))
        self.x, self.y, self.post = args["x_out"], None, None
        return 3, args

    def norm_gemv(self, gain: Tensor, w: Tensor, bias: Optional[Tensor] = None) -> Tensor:
        """``W norm(x) + bias``."""
        out = torch.empty((self.x.shape[0], w.shape[0]), dtype=w.dtype, device=w.device)
        kind, args = self._front(gain)
        _gemv(kind, 0, w, bias=bias, out=out, **args)
        return out

    def norm_gemv_f32(self, gain: Tensor, w: Tensor) -> Tensor:
        """``W norm(x)`` in fp32 (the vocabulary projection)."""
        out = torch.empty((self.x.shape[0], w.shape[0]), dtype=torch.float32, device=w.device)
        kind, args = self._front(gain)
        _gemv(kind, 1, w, res=out, **args)
        return out

    def norm_gemv_glu(self, gain: Tensor, w: Tensor, limit: float) -> Tensor:
        """``clamped_glu`` of the two halves of ``W norm(x)``; ``w [2F, K]`` = gate rows | up rows."""
        out = torch.empty((self.x.shape[0], w.shape[0] // 2), dtype=w.dtype, device=w.device)
        kind, args = self._front(gain)
        _gemv(kind, 3, w, limit=limit, out=out, **args)
        return out

    def norm_route(self, gain: Tensor, w: Tensor, routers: int) -> Tuple[Tensor, Tensor, Tensor]:
        """From ``norm(x)`` (there must be a pending output): a router's logits (fp32, ``w``'s first rows), ``silu(gate) * up``
        of the other rows, and the normed rows themselves."""
        M, (N, K) = self.x.shape[0], w.shape
        z = torch.empty((M, routers), dtype=torch.float32, device=w.device)
        act = torch.empty((M, (N - routers) // 2), dtype=w.dtype, device=w.device)
        h = torch.empty((M, K), dtype=w.dtype, device=w.device)
        kind, args = self._front(gain)
        _gemv(kind, 4, w, routers=routers, res=z, out=act, h_out=h, **args)
        return z, act, h

    def settled(self) -> Tensor:
        """The stream with the pending output added, as a tensor of its own."""
        x = self.x.clone()
        if self.y is not None:
            add_rmsnorm(x, self.y, self.mult, None, self.eps, torch.float32, norm=False, post=self.post)
        return x

    def rows(self, want) -> None:
        self.x = self.x[want].contiguous()
        self.y = None if self.y is None else self.y[want].contiguous()


def norm_gemv(x: Tensor, gain: Tensor, eps: float, w: Tensor, bias: Optional[Tensor] = None, w0: float = 1.0) -> Tensor:
    """``W (rms(x) * (w0 + gain)) + bias`` for a few rows of the fp32 stream ``x [M, K]``."""
    return Stream(x, eps, w0, 1.0).norm_gemv(gain, w, bias)


def norm_gemv_f32(x: Tensor, gain: Tensor, eps: float, w: Tensor, w0: float = 1.0) -> Tensor:
    """The same without bias, stored in fp32."""
    return Stream(x, eps, w0, 1.0).norm_gemv_f32(gain, w)


def norm_gemv_glu(x: Tensor, gain: Tensor, eps: float, w: Tensor, limit: float, w0: float = 1.0) -> Tensor:
    """``clamped_glu`` of the two halves of the product."""
    return Stream(x, eps, w0, 1.0).norm_gemv_glu(gain, w, limit)


def _fp32_rows(res: Tensor, M: int, N: int) -> Tensor:
    if res.dtype != torch.float32 or res.shape != (M, N) or not res.is_contiguous():
        raise ValueError("the residual stream must be contiguous float32 [M, N]")
    return res


def gemv_residual(x: Tensor, w: Tensor, mult: float, res: Tensor) -> None:
    """``res += mult * (W x)`` in the fp32 stream ``res [M, N]``."""
    _gemv(0, 2, w, x=x, ldx=x.stride(0), mult=mult, res=_fp32_rows(res, x.shape[0], w.shape[0]))


def gemv_f32(x: Tensor, w: Tensor) -> Tensor:
    """``W x`` in fp32."""
    out = torch.empty((x.shape[0], w.shape[0]), dtype=torch.float32, device=w.device)
    _gemv(0, 1, w, x=x, ldx=x.stride(0), res=out)
    return out


def row_norm_gemv(x: Tensor, o_x: int, gain: Tensor, eps: float, w: Tensor) -> Tensor:
    """``W (rms(x) * gain)`` of the columns of ``x`` from ``o_x`` on, as many as W has."""
    out = torch.empty((x.shape[0], w.shape[0]), dtype=w.dtype, device=w.device)
    _gemv(4, 0, w, x=x, ldx=x.stride(0), o_x=o_x, gain=gain, eps=eps, out=out)
    return out


def gated_norm_gemv_residual(y: Tensor, proj: Tensor, o_z: int, gain: Tensor, eps: float, groups: int, w: Tensor, mult: float,
                             res: Tensor) -> None:
    """``gated_group_norm`` and ``gemv_residual`` in one launch."""
    _gemv(2, 2, w, x=proj, ldx=proj.stride(0), o_x=o_z, xf=y, gain=gain, eps=eps, groups=groups, mult=mult,
          res=_fp32_rows(res, y.shape[0], w.shape[0]))


def norm_gate_gemv_f32(y: Tensor, proj: Tensor, o_z: int, gain: Tensor, eps: float, w: Tensor) -> Tensor:
    """``norm_gate`` and a product in fp32 in one launch."""
    out = torch.empty((y.shape[0], w.shape[0]), dtype=torch.float32, device=w.device)
    _gemv(5, 1, w, x=proj, ldx=proj.stride(0), o_x=o_z, xf=y, gain=gain, eps=eps, res=out)
    return out


# ------------------------------------------------------------------------------------------------ convolution state
def _ring(ring: Tensor, C: int, taps: int, dtype) -> None:
    if ring.dim() != 3 or tuple(ring.shape[1:]) != (taps, C) or ring.dtype != dtype or not ring.is_contiguous():
        raise ValueError(f"the convolution ring must be contiguous {dtype} [slots, {taps}, {C}], got {tuple(ring.shape)}")


def conv_silu(proj: Tensor, o_in: int, w: Tensor, bias: Optional[Tensor], ring: Tensor, b: Batch) -> Tensor:
    """Causal convolution (``w [C, taps]``) and SiLU of ``C`` columns of ``proj``; fp32 ``[M, C]``."""
    _need_gpu(proj, w, bias, ring, b.pos)
    C, taps = w.shape
    _batch(b, proj.shape[0])
    _ring(ring, C, taps, proj.dtype)
    _vec(w, C * taps, "w")
    _vec(bias, C, "bias")
    if o_in + C > proj.shape[1]:
        raise ValueError("conv_silu: channels outside the projection")
    out = torch.empty((proj.shape[0], C), dtype=torch.float32, device=proj.device)
    _call("aqs_conv_silu", proj.device, _p(proj, o_in), proj.stride(0), _DT[proj.dtype], _p(w), _p(bias), _p(ring), _p(b.slots),
          _p(b.pos), _p(out), b.B, b.S, C, taps, _stream(proj))
    return out


def conv_push(proj: Tensor, o_in: int, C: int, taps: int, ring: Tensor, b: Batch) -> None:
    """Keep the last ``taps - 1`` inputs; after everything that reads the ring's old content."""
    _batch(b, proj.shape[0])
    _ring(ring, C, taps, proj.dtype)
    _call("aqs_conv_push", proj.device, _p(proj, o_in), proj.stride(0), _DT[proj.dtype], _p(ring), _p(b.slots), _p(b.pos), b.B,
          b.S, C, taps, _stream(proj))


# ------------------------------------------------------------------------------------------------ recurrences
def _state(s: Tensor, *dims) -> None:
    if s.dtype != torch.float32 or tuple(s.shape[1:]) != dims or not s.is_contiguous():
        raise ValueError(f"the recurrent state must be contiguous float32 [slots, {dims}], got {tuple(s.shape)}")


def delta_prep(proj: Tensor, o_qkv: int, raw: Tensor, o_beta: int, conv_w: Tensor, ring: Tensor, a_log: Tensor, dt_bias: Tensor,
               H: int, G: int, D: int, E: int, b: Batch):
    """Inputs of the delta rule: ``(q, k [M, G, D], v [M, H, E], decay [M, H, D], beta [M, H])`` in fp32."""
    _need_gpu(proj, raw, conv_w, ring, a_log, dt_bias)
    M, C, taps, dev = proj.shape[0], 2 * G * D + H * E, conv_w.shape[1], proj.device
    _batch(b, M)
    _ring(ring, C, taps, proj.dtype)
    _vec(conv_w, C * taps, "conv_w")
    _vec(a_log, H, "a_log")
    _vec(dt_bias, H * D, "dt_bias")
    _rows2(raw, "raw", proj.dtype)
    if raw.shape != (M, H * D) or o_qkv + C > proj.shape[1] or o_beta + H > proj.shape[1]:
        raise ValueError("delta_prep: shapes do not fit")
    q = torch.empty((M, G, D), dtype=torch.float32, device=dev)
    k = torch.empty_like(q)
    v = torch.empty((M, H, E), dtype=torch.float32, device=dev)
    decay = torch.empty((M, H, D), dtype=torch.float32, device=dev)
    beta = torch.empty((M, H), dtype=torch.float32, device=dev)
    _call("aqs_delta_prep", dev, _p(proj, o_qkv), proj.stride(0), _p(raw), raw.stride(0), _p(proj, o_beta), proj.stride(0),
          _DT[proj.dtype], _p(conv_w), _p(ring), _p(b.slots), _p(b.pos), _p(a_log), _p(dt_bias), _p(q), _p(k), _p(v), _p(decay),
          _p(beta), b.B, b.S, H, G, D, E, taps, _stream(proj))
    return q, k, v, decay, beta


def delta_scan(q: Tensor, k: Tensor, v: Tensor, decay: Tensor, beta: Tensor, state: Tensor, b: Batch) -> Tensor:
    """The gated delta rule over the new tokens; ``state [slots, H, E, D]`` is carried on.  fp32 ``[M, H, E]``."""
    _need_gpu(q, k, v, decay, beta, state)
    M, G, D = q.shape
    H, E = v.shape[1:]
    _batch(b, M)
    _state(state, H, E, D)
    for t, n in ((q, M * G * D), (k, M * G * D), (v, M * H * E), (decay, M * H * D), (beta, M * H)):
        _vec(t, n, "delta_scan input")
    out = torch.empty((M, H, E), dtype=torch.float32, device=q.device)
    _call("aqs_delta_scan", q.device, _p(q), _p(k), _p(v), _p(decay), _p(beta), _p(state), _p(b.slots), _p(b.pos), _p(out), b.B,
          b.S, H, G, D, E, _stream(q))
    return out


STEP_MAX = 256    # rows and columns of a head's state in the one-token kernels
CHUNKED_MIN = 96  # new tokens per sequence from which the chunked kernels are the faster ones


def chunked_ok(rows: int, taps: int) -> bool:
    """Whether the chunked recurrences serve a state of ``rows`` rows behind a convolution of ``taps`` taps."""
    return bool(_abi.load_seq().aqs_chunked_ok(rows, taps))


def delta_chunked(proj: Tensor, o_qkv: int, raw: Tensor, o_beta: int, conv_w: Tensor, ring: Tensor, a_log: Tensor, dt_bias: Tensor,
                  state: Tensor, H: int, G: int, D: int, E: int, b: Batch) -> Tensor:
    """``delta_prep`` and ``delta_scan`` in chunks of 64 tokens on the fp32 matrix cores.  fp32 ``[M, H, E]``."""
    _need_gpu(proj, raw, conv_w, ring, a_log, dt_bias, state)
    M, C, taps, dev = proj.shape[0], 2 * G * D + H * E, conv_w.shape[1], proj.device
    _batch(b, M)
    _ring(ring, C, taps, proj.dtype)
    _state(state, H, E, D)
    _vec(conv_w, C * taps, "conv_w")
    _vec(a_log, H, "a_log")
    _vec(dt_bias, H * D, "dt_bias")
    _rows2(raw, "raw", proj.dtype)
    if raw.shape != (M, H * D) or o_qkv + C > proj.shape[1] or o_beta + H > proj.shape[1]:
        raise ValueError("delta_chunked: shapes do not fit")
    n = int(_abi.load_seq().aqs_delta_chunked_ws(b.B, b.S, H, D, E))
    ws = torch.empty(n, dtype=torch.float32, device=dev)
    out = torch.empty((M, H, E), dtype=torch.float32, device=dev)
    _call("aqs_delta_chunked", dev, _p(proj, o_qkv), proj.stride(0), _p(raw), raw.stride(0), _p(proj, o_beta), proj.stride(0),
          _DT[proj.dtype], _p(conv_w), _p(ring), _p(b.slots), _p(b.pos), _p(a_log), _p(dt_bias), _p(ws), n, _p(state), _p(out),
          b.B, b.S, H, G, D, E, taps, _stream(proj))
    return out


def _step_constants(H: int, dt_bias, a_log, skip, decay) -> None:
    for t in (dt_bias, a_log, skip, decay):
        _vec(t, H, "per-head constants")
    if decay is None and (dt_bias is None or a_log is None):
        raise ValueError("step sizes need dt_bias and a_log")


def ssd_chunked(proj: Tensor, o_xbc: int, o_dt: int, conv_w: Tensor, conv_b: Tensor, ring: Tensor, dt_bias: Optional[Tensor],
                a_log: Optional[Tensor], skip: Optional[Tensor], state: Tensor, H: int, G: int, N: int, P: int, b: Batch,
                decay: Optional[Tensor] = None) -> Tensor:
    """``conv_silu`` and ``ssd_scan`` in chunks of 64 tokens on the fp32 matrix cores.  fp32 ``[M, H * P]``."""
    _need_gpu(proj, conv_w, conv_b, ring, dt_bias, a_log, skip, state, decay)
    M, C, taps, dev = proj.shape[0], H * P + 2 * G * N, conv_w.shape[1], proj.device
    _batch(b, M)
    _ring(ring, C, taps, proj.dtype)
    _state(state, H, P, N)
    _vec(conv_w, C * taps, "conv_w")
    _vec(conv_b, C, "conv_b")
    _step_constants(H, dt_bias, a_log, skip, decay)
    if o_xbc + C > proj.shape[1] or (decay is None and o_dt + H > proj.shape[1]):
        raise ValueError("ssd_chunked: shapes do not fit")
    n = int(_abi.load_seq().aqs_ssd_chunked_ws(b.B, b.S, H, G, N))
    ws = torch.empty(n, dtype=torch.float32, device=dev)
    out = torch.empty((M, H * P), dtype=torch.float32, device=dev)
    _call("aqs_ssd_chunked", dev, _p(proj, o_xbc), proj.stride(0), _p(proj, o_dt), proj.stride(0), _DT[proj.dtype], _p(conv_w),
          _p(conv_b), _p(ring), _p(b.slots), _p(b.pos), _p(dt_bias), _p(a_log), _p(skip), _p(decay), _p(ws), n, _p(state), _p(out), b.B,
          b.S, H, G, N, P, taps, _stream(proj))
    return out


def delta_step(proj: Tensor, o_qkv: int, o_beta: int, o_a1: int, o_g1: int, conv_w: Tensor, ring: Tensor, a2: Tensor, g2: Tensor,
               a_log: Tensor, dt_bias: Tensor, norm: Tensor, eps: float, scale: float, state: Tensor, out: Tensor, H: int, G: int,
               D: int, E: int, b: Batch) -> None:
    """One token per sequence, from the projection's row to the normed and gated heads ``out [B, H * E]``."""
    _need_gpu(proj, conv_w, ring, a2, g2, state, out)
    C, taps = 2 * G * D + H * E, conv_w.shape[1]
    _batch(b, proj.shape[0])
    _ring(ring, C, taps, proj.dtype)
    _state(state, H, E, D)
    _rows2(out, "out", proj.dtype)
    _vec(conv_w, C * taps, "conv_w")
    _vec(a_log, H, "a_log")
    _vec(dt_bias, H * D, "dt_bias")
    _vec(norm, E, "norm")
    if b.S != 1 or out.shape != (b.B, H * E) or a2.shape[0] != H * D or g2.shape[0] != H * E or a2.dtype != proj.dtype \
            or g2.dtype != proj.dtype or not a2.is_contiguous() or not g2.is_contiguous():
        raise ValueError("delta_step: shapes do not fit")
    _call("aqs_delta_step", proj.device, _p(proj), proj.stride(0), o_qkv, o_beta, o_a1, o_g1, _DT[proj.dtype], _p(conv_w), _p(ring),
          _p(b.slots), _p(b.pos), _p(a2), a2.shape[1], _p(g2), g2.shape[1], _p(a_log), _p(dt_bias), _p(norm), float(eps),
          float(scale), _p(state), _p(out), out.stride(0), b.B, H, G, D, E, taps, _stream(proj))


def ssd_scan(xbc: Tensor, proj: Tensor, o_dt: int, dt_bias: Optional[Tensor], a_log: Optional[Tensor], skip: Optional[Tensor],
             state: Tensor, H: int, G: int, N: int, P: int, b: Batch, decay: Optional[Tensor] = None) -> Tensor:
    """The state-space recurrence over the new tokens; ``xbc`` from ``conv_silu``.  fp32 ``[M, H * P]``.  ``decay [H]``: constant
    decays and step size 1 (linear attention: x, B and C are its v, k and q)."""
    _need_gpu(xbc, proj, dt_bias, a_log, skip, state, decay)
    M = xbc.shape[0]
    _batch(b, M)
    _state(state, H, P, N)
    _vec(xbc, M * (H * P + 2 * G * N), "xbc")
    _step_constants(H, dt_bias, a_log, skip, decay)
    if proj.shape[0] != M or (decay is None and o_dt + H > proj.shape[1]):
        raise ValueError("ssd_scan: shapes do not fit")
    out = torch.empty((M, H * P), dtype=torch.float32, device=xbc.device)
    _call("aqs_ssd_scan", xbc.device, _p(xbc), _p(proj, o_dt), proj.stride(0), _DT[proj.dtype], _p(dt_bias), _p(a_log), _p(skip),
          _p(decay), _p(state), _p(b.slots), _p(b.pos), _p(out), b.B, b.S, H, G, N, P, _stream(xbc))
    return out


def ssd_step(proj: Tensor, o_xbc: int, o_dt: int, conv_w: Tensor, conv_b: Tensor, ring: Tensor, dt_bias: Optional[Tensor],
             a_log: Optional[Tensor], skip: Optional[Tensor], state: Tensor, H: int, G: int, N: int, P: int, b: Batch,
             decay: Optional[Tensor] = None) -> Tensor:
    """One token per sequence: convolution, step size, recurrence.  fp32 ``[B, H * P]``, before gate and norm."""
    _need_gpu(proj, conv_w, conv_b, ring, state, decay)
    C, taps = H * P + 2 * G * N, conv_w.shape[1]
    _batch(b, proj.shape[0])
    _ring(ring, C, taps, proj.dtype)
    _state(state, H, P, N)
    _vec(conv_w, C * taps, "conv_w")
    _vec(conv_b, C, "conv_b")
    _step_constants(H, dt_bias, a_log, skip, decay)
    if b.S != 1:
        raise ValueError("ssd_step takes one token per sequence")
    y = torch.empty((b.B, H * P), dtype=torch.float32, device=proj.device)
    _call("aqs_ssd_step", proj.device, _p(proj), proj.stride(0), o_xbc, o_dt, _DT[proj.dtype], _p(conv_w), _p(conv_b), _p(ring),
          _p(b.slots), _p(b.pos), _p(dt_bias), _p(a_log), _p(skip), _p(decay), _p(state), _p(y), b.B, H, G, N, P, taps, _stream(proj))
    return y


# ------------------------------------------------------------------------------------------------ windowed attention
class WindowAttnSpec(NamedTuple):
    """Sizes and constants of a windowed attention."""
    H: int
    G: int
    D: int
    E: int
    window: int
    scale: float
    rot: int
    eps: float


def _pages(kc: Tensor, vc: Tensor, s: WindowAttnSpec, dtype) -> None:
    if kc.dim() != 4 or vc.dim() != 4 or kc.shape[:2] != vc.shape[:2] or tuple(kc.shape[2:]) != (s.G, s.D) \
            or tuple(vc.shape[2:]) != (s.G, s.E) or kc.dtype != dtype or vc.dtype != dtype \
            or not (kc.is_contiguous() and vc.is_contiguous()):
        raise ValueError(f"caches must be contiguous {dtype} [pages, page, {s.G}, {s.D} / {s.E}], got {tuple(kc.shape)}, {tuple(vc.shape)}")


def _rotary(cs: Tensor, s: WindowAttnSpec) -> None:
    if cs.dtype != torch.float32 or cs.dim() != 3 or tuple(cs.shape[1:]) != (s.rot // 2, 2) or not cs.is_contiguous():
        raise ValueError(f"the rotary table must be contiguous float32 [positions, {s.rot // 2}, 2], got {tuple(cs.shape)}")


def attn_prep(proj: Tensor, o_q: int, o_k: int, o_v: int, q_norm: Tensor, k_norm: Tensor, cs: Tensor, kc: Tensor, vc: Tensor,
              s: WindowAttnSpec, b: Batch) -> Tensor:
    """Head norms and rotation of q and k; k and v into their page slots.  Returns ``q [M, H, D]``."""
    _need_gpu(proj, q_norm, k_norm, cs, kc, vc)
    _batch(b, proj.shape[0])
    _pages(kc, vc, s, proj.dtype)
    _rotary(cs, s)
    _vec(q_norm, s.D, "q_norm")
    _vec(k_norm, s.D, "k_norm")
    q = torch.empty((proj.shape[0], s.H, s.D), dtype=proj.dtype, device=proj.device)
    _call("aqs_attn_prep", proj.device, _p(proj), proj.stride(0), o_q, o_k, o_v, _DT[proj.dtype], _p(q_norm), _p(k_norm), s.eps,
          _p(cs), cs.shape[0], s.rot, _p(b.pos), _p(b.table), b.table.shape[1], kc.shape[1], kc.shape[0], _p(q), _p(kc), _p(vc),
          b.B, b.S, s.H, s.G, s.D, s.E, _stream(proj))
    return q


def attn_window(q: Tensor, kc: Tensor, vc: Tensor, proj: Tensor, o_gate: int, out_scale: float, s: WindowAttnSpec, b: Batch,
                out: Tensor, simple: bool = False) -> None:
    """The new tokens over their windows; ``out [M, H * E]`` gated per head by ``proj``'s columns from ``o_gate`` on
    (none for ``o_gate < 0``) and scaled."""
    _need_gpu(q, kc, vc, proj, out)
    _batch(b, q.shape[0])
    _pages(kc, vc, s, q.dtype)
    _rows2(out, "out", q.dtype)
    if tuple(q.shape[1:]) != (s.H, s.D) or not q.is_contiguous() or out.shape != (q.shape[0], s.H * s.E) \
            or (o_gate >= 0 and o_gate + s.H > proj.shape[1]):
        raise ValueError("attn_window: shapes do not fit")
    _call("aqs_attn_window", q.device, _p(q), _p(kc), _p(vc), _DT[q.dtype], s.scale, s.window,
          _p(proj, o_gate) if o_gate >= 0 else None, proj.stride(0), float(out_scale), _p(b.pos), _p(b.table), b.table.shape[1],
          kc.shape[1], kc.shape[0], _p(out), out.stride(0), b.B, b.S, s.H, s.G, s.D, s.E, int(simple), _stream(q))


def attn_decode_ok(s: WindowAttnSpec, page: int) -> bool:
    return bool(_abi.load_seq().aqs_attn_decode_ok(s.D, s.E, page))


def attn_decode(proj: Tensor, o_q: int, o_k: int, o_v: int, o_gate: int, q_norm: Tensor, k_norm: Tensor, cs: Tensor, kc: Tensor,
                vc: Tensor, out_scale: float, s: WindowAttnSpec, b: Batch, out: Tensor) -> None:
    """``attn_prep`` and ``attn_window`` for one token per sequence."""
    _need_gpu(proj, q_norm, k_norm, cs, kc, vc, out)
    _batch(b, proj.shape[0])
    _pages(kc, vc, s, proj.dtype)
    _rotary(cs, s)
    _rows2(out, "out", proj.dtype)
    _vec(q_norm, s.D, "q_norm")
    _vec(k_norm, s.D, "k_norm")
    if b.S != 1 or out.shape != (b.B, s.H * s.E):
        raise ValueError("attn_decode: shapes do not fit")
    n = int(_abi.load_seq().aqs_attn_decode_slices(s.window, b.table.shape[1] * kc.shape[1]))
    part = torch.empty((b.B, s.H, n, s.E + 4), dtype=torch.float32, device=proj.device)
    _call("aqs_attn_decode", proj.device, _p(proj), proj.stride(0), o_q, o_k, o_v, o_gate, _DT[proj.dtype], _p(q_norm), _p(k_norm),
          s.eps, _p(cs), cs.shape[0], s.rot, s.scale, s.window, float(out_scale), _p(b.pos), _p(b.table), b.table.shape[1],
          kc.shape[1], kc.shape[0], _p(kc), _p(vc), _p(part), n, _p(out), out.stride(0), b.B, s.H, s.G, s.D, s.E, _stream(proj))


# ------------------------------------------------------------------------------------------------ latent attention
class LatentSpec(NamedTuple):
    """Sizes and constants of a latent attention: H heads of ``dim`` unrotated and ``rot`` rotated key elements (the first
    ``rd`` of them in pairs) and E value elements, latents of QR (queries) and R (keys and values)."""
    H: int
    dim: int
    rot: int
    rd: int
    E: int
    QR: int
    R: int
    window: int
    scale: float
    eps: float


def _latent_pages(kc: Tensor, s: LatentSpec, dtype) -> None:
    if kc.dim() != 4 or tuple(kc.shape[2:]) != (1, s.R + s.rot) or kc.dtype != dtype or not kc.is_contiguous():
        raise ValueError(f"the cache must be contiguous {dtype} [pages, page, 1, {s.R + s.rot}], got {tuple(kc.shape)}")


def _latent_rotary(cs: Tensor, s: LatentSpec) -> None:
    if cs.dtype != torch.float32 or cs.dim() != 3 or tuple(cs.shape[1:]) != (s.rd // 2, 2) or not cs.is_contiguous():
        raise ValueError(f"the rotary table must be contiguous float32 [positions, {s.rd // 2}, 2], got {tuple(cs.shape)}")


def latent_rows(s: LatentSpec, b: Batch, capacity: int) -> int:
    """Packed rows per sequence: the blocks of 64 positions from a window's first to the last new token."""
    if b.starts is None:
        return min((s.window + b.S + 125) // 64, (capacity + 63) // 64) * 64
    return max((p + b.S - 1) // 64 - max(p - s.window + 1, 0) // 64 + 1 for p in b.starts) * 64


def latent_prep(proj: Tensor, o_q: int, o_kv: int, q_norm: Tensor, kv_norm: Tensor, cs: Tensor, kc: Tensor, s: LatentSpec,
                b: Batch) -> Tuple[Tensor, Tensor]:
    """Normed query latents ``[M, QR]``; the new tokens' cache rows into the pages; and the rows that their windows reach,
    ``[B * rows, R + rot]``."""
    _need_gpu(proj, q_norm, kv_norm, cs, kc)
    M, DK = proj.shape[0], s.R + s.rot
    _batch(b, M)
    _rows2(proj, "proj")
    _latent_pages(kc, s, proj.dtype)
    _latent_rotary(cs, s)
    _vec(q_norm, s.QR, "q_norm")
    _vec(kv_norm, s.R, "kv_norm")
    rows = latent_rows(s, b, b.table.shape[1] * kc.shape[1])
    cq = torch.empty((M, s.QR), dtype=proj.dtype, device=proj.device)
    packed = torch.empty((b.B * rows, DK), dtype=proj.dtype, device=proj.device)
    _call("aqs_latent_prep", proj.device, _p(proj), proj.stride(0), o_q, o_kv, _DT[proj.dtype], _p(q_norm), _p(kv_norm), s.eps, _p(cs),
          cs.shape[0], _p(b.pos), _p(b.table), b.table.shape[1], kc.shape[1], kc.shape[0], s.window, _p(cq), _p(kc), _p(packed), rows,
          b.B, b.S, s.QR, s.R, s.rot, s.rd, _stream(proj))
    return cq, packed


def latent_rotate(q: Tensor, cs: Tensor, s: LatentSpec, b: Batch) -> None:
    """The rotated part of every head of ``q [M, H * (dim + rot)]``, in place."""
    _need_gpu(q, cs)
    _batch(b, q.shape[0])
    _latent_rotary(cs, s)
    if q.shape[1] != s.H * (s.dim + s.rot) or not q.is_contiguous():
        raise ValueError("latent_rotate: q must be contiguous [M, H * (dim + rot)]")
    _call("aqs_latent_rotate", q.device, _p(q), _DT[q.dtype], _p(cs), cs.shape[0], _p(b.pos), b.B, b.S, s.H, s.dim, s.rot, s.rd, _stream(q))


def latent_window(q: Tensor, kv: Tensor, packed: Tensor, proj: Tensor, o_gate: int, s: LatentSpec, b: Batch, out: Tensor,
                  simple: bool = False) -> None:
    """The new tokens over their windows: keys and values of all heads ``kv [B * rows, H * (dim + E)]``, rotated key parts from
    ``packed``; ``out [M, H * E]`` gated by ``proj``'s columns from ``o_gate`` on, element by element."""
    _need_gpu(q, kv, packed, proj, out)
    _batch(b, q.shape[0])
    _rows2(out, "out", q.dtype)
    rows = packed.shape[0] // b.B
    if q.shape[1] != s.H * (s.dim + s.rot) or not q.is_contiguous() or kv.shape != (packed.shape[0], s.H * (s.dim + s.E)) \
            or packed.shape != (b.B * rows, s.R + s.rot) or not packed.is_contiguous() or kv.dtype != q.dtype or packed.dtype != q.dtype \
            or proj.dtype != q.dtype or out.shape != (q.shape[0], s.H * s.E) or o_gate + s.H * s.E > proj.shape[1]:
        raise ValueError("latent_window: shapes do not fit")
    _rows2(kv, "kv")
    _call("aqs_latent_window", q.device, _p(q), _p(kv), kv.stride(0), _p(packed), packed.stride(0), s.R, _DT[q.dtype], s.scale, s.window,
          _p(proj, o_gate), proj.stride(0), _p(b.pos), rows, _p(out), out.stride(0), b.B, b.S, s.H, s.dim, s.rot, s.E, int(simple), _stream(q))


def latent_decode_ok(s: LatentSpec, B: int, page: int) -> bool:
    return bool(_abi.load_seq().aqs_latent_decode_ok(B, s.dim, s.rot, s.R, s.E, page))


def latent_decode(proj: Tensor, o_kv: int, o_gate: int, q: Tensor, uk: Tensor, uv: Tensor, kv_norm: Tensor, cs: Tensor, kc: Tensor,
                  s: LatentSpec, b: Batch, out: Tensor) -> None:
    """One token per sequence from the projection's row and its queries ``q [B, H * (dim + rot)]`` (not yet rotated) to the gated
    heads: ``latent_prep`` and ``latent_window``, with the key and value factors moved to the query and the output."""
    _need_gpu(proj, q, uk, uv, kv_norm, cs, kc, out)
    _batch(b, proj.shape[0])
    _latent_pages(kc, s, proj.dtype)
    _latent_rotary(cs, s)
    _rows2(out, "out", proj.dtype)
    _vec(kv_norm, s.R, "kv_norm")
    if b.S != 1 or out.shape != (b.B, s.H * s.E) or q.shape != (b.B, s.H * (s.dim + s.rot)) or not q.is_contiguous() \
            or uk.shape != (s.H * s.dim, s.R) or uv.shape != (s.H * s.E, s.R) or not (uk.is_contiguous() and uv.is_contiguous()) \
            or any(t.dtype != proj.dtype for t in (q, uk, uv)):
        raise ValueError("latent_decode: shapes do not fit")
    n = int(_abi.load_seq().aqs_latent_decode_slices(s.window, b.table.shape[1] * kc.shape[1]))
    qa = torch.empty((b.B, s.H, s.R + s.rot), dtype=proj.dtype, device=proj.device)
    part = torch.empty((b.B, s.H, n, s.R + 4), dtype=torch.float32, device=proj.device)
    _call("aqs_latent_decode", proj.device, _p(proj), proj.stride(0), o_kv, o_gate, _p(q), _p(uk), _p(uv), _DT[proj.dtype], _p(kv_norm),
          s.eps, _p(cs), cs.shape[0], s.scale, s.window, _p(b.pos), _p(b.table), b.table.shape[1], kc.shape[1], kc.shape[0], _p(kc), _p(qa),
          _p(part), n, _p(out), out.stride(0), b.B, s.H, s.dim, s.rot, s.rd, s.R, s.E, _stream(proj))


# ------------------------------------------------------------------------------------------------ routed experts
def moe_route(h: Tensor, router: Tensor, top: int) -> Tuple[Tensor, Tensor]:
    """``(experts int32 [M, top], scores [M, top])``: the ``top`` largest of ``sigmoid(router h)`` of every row."""
    _need_gpu(h, router)
    _rows2(h, "h", router.dtype)
    M, (Ex, K) = h.shape[0], router.shape
    if h.shape[1] != K or not router.is_contiguous():
        raise ValueError("the router must be contiguous [experts, K]")
    ids = torch.empty((M, top), dtype=torch.int32, device=h.device)
    scores = torch.empty((M, top), dtype=torch.float32, device=h.device)
    _call("aqs_moe_route", h.device, _p(h), h.stride(0), _DT[h.dtype], _p(router), _p(ids), _p(scores), M, K, Ex, top, _stream(h))
    return ids, scores


def moe_experts(h: Tensor, ids: Tensor, scores: Tensor, gate_up: Tensor, down: Tensor) -> Routed:
    """The chosen experts on the rows scaled by their scores: ``gate_up [Ex, 2F, K]`` (gate | up), ``down [Ex, K, F]``."""
    _need_gpu(h, ids, scores, gate_up, down)
    _rows2(h, "h", gate_up.dtype)
    (M, K), top = h.shape, ids.shape[1]
    Ex, F = gate_up.shape[0], gate_up.shape[1] // 2
    if gate_up.shape != (Ex, 2 * F, K) or down.shape != (Ex, K, F) or not (gate_up.is_contiguous() and down.is_contiguous()) \
            or down.dtype != h.dtype or ids.shape != (M, top) or scores.shape != (M, top) or ids.dtype != torch.int32 \
            or scores.dtype != torch.float32 or not (ids.is_contiguous() and scores.is_contiguous()):
        raise ValueError("moe_experts: shapes do not fit")
    lib, A, dev = _abi.load_seq(), M * top, h.device
    tile = int(lib.aqs_moe_tile(_DT[h.dtype], A, Ex, K, F))
    if tile != 64 and (h.stride(0) % 8 or h.data_ptr() % 16):
        h = h.contiguous()
    n = int(lib.aqs_moe_tiles(A, Ex, tile))
    rows = torch.empty(A, dtype=torch.int32, device=dev)
    slots = torch.empty((M, top), dtype=torch.int32, device=dev)
    tiles = torch.empty((n, 4), dtype=torch.int32, device=dev)
    act = torch.empty((A, F), dtype=h.dtype, device=dev)
    out = torch.empty((A, K), dtype=h.dtype, device=dev)
    _call("aqs_moe_sort", dev, _p(ids), A, Ex, tile, _p(rows), _p(slots), _p(tiles), n, _stream(h))
    _call("aqs_moe_product", dev, 1, _p(h), h.stride(0), _DT[h.dtype], _p(gate_up), _p(tiles), n, tile, _p(rows), _p(scores), A, top,
          _p(act), 2 * F, K, _stream(h))
    _call("aqs_moe_product", dev, 0, _p(act), F, _DT[h.dtype], _p(down), _p(tiles), n, tile, _p(rows), None, A, top, _p(out), K, F,
          _stream(h))
    return Routed(out, slots)


def moe_step_ok(M: int, K: int, F: int, Fs: int, Ex: int, top: int) -> bool:
    return bool(_abi.load_seq().aqs_moe_step_ok(M, K, F, Fs, Ex, top))


def moe_step(h: Tensor, z: Tensor, top: int, gate_up: Tensor, down: Tensor, shared: Optional[Tensor] = None,
             shared_down: Optional[Tensor] = None) -> Tensor:
    """Up to 8 rows ``h`` with router logits ``z``: the chosen experts and ``shared_down shared``, added; fp32 ``[M, K]``."""
    _need_gpu(h, z, gate_up, down, shared, shared_down)
    M, K = h.shape
    Ex, F = gate_up.shape[0], gate_up.shape[1] // 2
    Fs = 0 if shared is None else shared.shape[1]
    if gate_up.shape != (Ex, 2 * F, K) or down.shape != (Ex, K, F) or z.shape != (M, Ex) or z.dtype != torch.float32 \
            or any(t.dtype != h.dtype or not t.is_contiguous() for t in (h, gate_up, down)) or not z.is_contiguous():
        raise ValueError("moe_step: shapes do not fit")
    if Fs and (shared.shape != (M, Fs) or shared_down.shape != (K, Fs) or not (shared.is_contiguous() and shared_down.is_contiguous())
               or shared.dtype != h.dtype or shared_down.dtype != h.dtype):
        raise ValueError("moe_step: the shared expert's shapes do not fit")
    act = torch.empty((M * top, F), dtype=h.dtype, device=h.device)
    y = torch.empty((M, K), dtype=torch.float32, device=h.device)
    _call("aqs_moe_step_up", h.device, _p(h), _p(z), _DT[h.dtype], _p(gate_up), _p(act), M, K, F, Ex, top, _stream(h))
    _call("aqs_moe_step_down", h.device, _p(z), _p(act), _DT[h.dtype], _p(down), _p(shared), _p(shared_down), _p(y), M, K, F, Fs, Ex, top,
          _stream(h))
    return y
