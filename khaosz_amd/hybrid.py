"""Decoders whose layers mix linear recurrences and windowed attention, configured layer by layer.

``Rudilix``: embedding, pre-norm layers ``x += m mixer(norm(x)); x += m ff(norm(x))`` with mixers of three kinds
(``mamba2``, ``channel_delta``, and ``parallel``: windowed attention beside a channel delta rule), norms with their
weight around zero, clamped GLU feed-forwards, an untied vocabulary projection.  Which mixer a layer has, every size
and every constant come from the configuration.

The residual stream is fp32 throughout; weights and activations are bf16 or fp32.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional, Sequence

import torch
import torch.nn as nn
import torch.nn.functional as F
from torch import Tensor

from . import seq_ops
from .mixers import ChannelDeltaMixer, ClampedGLU, Mamba2Mixer, MixerBlock, WindowAttention, _param
from .registry import register_model
from .seq_ops import Batch


@dataclass
class HybridConfig:
    """The fields of config.json.  ``layers[i]``: ``type``, the mixer's sizes ``mixer``, and ``mlp`` (or None)."""

    vocab: int
    width: int
    layers: List[Dict[str, Any]]
    norm_eps: float
    residual_mult: float = 1.0
    # ranks of the low-rank factors, by tensor name: no other field gives them, so they come from the tensors' shapes
    ranks: Dict[str, int] = field(default_factory=dict)

    @classmethod
    def from_dict(cls, d: Dict[str, Any], shapes: Optional[Dict[str, Sequence[int]]] = None) -> "HybridConfig":
        for i, layer in enumerate(d["layers"]):
            if layer["type"] not in LAYER_MIXERS:
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}, know {sorted(LAYER_MIXERS)}")
            mlp = layer.get("mlp")
            if mlp is not None and mlp["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
        ranks = {n: s[0] for n, s in (shapes or {}).items() if n.endswith((".a1", ".g1"))}
        return cls(int(d["vocab"]), int(d["width"]), d["layers"], float(d["norm"]["eps"]), float(d["residual_mult"]), ranks)


def _mamba2(cfg: HybridConfig, c, prefix: str, dtype, device):
    return [("", Mamba2Mixer(c, cfg.norm_eps, dtype, device), 1.0)]


def _delta(cfg: HybridConfig, c, prefix: str, dtype, device):
    ranks = []
    for n in ("a1", "g1"):
        if prefix + n not in cfg.ranks:
            raise ValueError(f"the rank of {prefix}{n} is not known: give it in ranks, or load from a checkpoint")
        ranks.append(int(cfg.ranks[prefix + n]))
    return [("", ChannelDeltaMixer(c, cfg.norm_eps, (ranks[0], ranks[1]), dtype, device), 1.0)]


def _parallel(cfg: HybridConfig, c, prefix: str, dtype, device):
    left = WindowAttention(c["left"], cfg.norm_eps, dtype, device)
    (_, right, _), = _delta(cfg, c["right"], prefix + "right.", dtype, device)
    return [("left.", left, c["left_scale"]), ("right.", right, c["right_scale"])]


LAYER_MIXERS = {"mamba2": _mamba2, "channel_delta": _delta, "parallel": _parallel}


class HybridLayer(nn.Module):
    def __init__(self, cfg: HybridConfig, index: int, dtype, device=None):
        super().__init__()
        layer = cfg.layers[index]
        self.prefix, self.eps, self.mult = f"l{index}.", cfg.norm_eps, cfg.residual_mult
        mixers = LAYER_MIXERS[layer["type"]](cfg, layer["mixer"], self.prefix + "mix.", dtype, device)
        self.norm1 = _param(cfg.width, device=device)
        self.mixer = MixerBlock(cfg.width, mixers, dtype, device)
        self.mlp = None
        if layer.get("mlp") is not None:
            self.norm2 = _param(cfg.width, device=device)
            self.mlp = ClampedGLU(cfg.width, layer["mlp"], dtype, device)

    def tensors(self) -> Dict[str, Tensor]:
        out = {self.prefix + "norm1": self.norm1}
        out.update({self.prefix + "mix." + n: t for n, t in self.mixer.tensors().items()})
        if self.mlp is not None:
            out[self.prefix + "norm2"] = self.norm2
            out.update({self.prefix + "mlp." + n: t for n, t in self.mlp.tensors().items()})
        return out

    def prompt(self, x: Tensor, y: Optional[Tensor], b: Batch, st, dtype) -> Tensor:
        """Adds the pending branch output ``y`` to the stream, runs the layer and returns its own pending output."""
        h = seq_ops.add_rmsnorm(x, y, self.mult, self.norm1, self.eps, dtype)
        y = self.mixer.prompt(h, b, st)
        if self.mlp is None:
            return y
        return self.mlp.prompt(seq_ops.add_rmsnorm(x, y, self.mult, self.norm2, self.eps, dtype))

    def step(self, x: Tensor, b: Batch, st) -> None:
        self.mixer.step(x, self.norm1, self.eps, b, st, self.mult)
        if self.mlp is not None:
            self.mlp.step(x, self.norm2, self.eps, self.mult)

    def step_ok(self, rows: int) -> bool:
        return self.mixer.step_ok(rows) and (self.mlp is None or self.mlp.step_ok(rows))


@register_model("Rudilix")
class HybridLM(nn.Module):
    """``forward`` runs new tokens of a batch of sequences on the state that earlier calls left."""

    config_class = HybridConfig
    mixed_positions = True  # sequences of one step may sit at different positions

    def __init__(self, config: HybridConfig, dtype: torch.dtype = torch.bfloat16, device=None):
        super().__init__()
        self.config, self.dtype = config, dtype
        self.embed = _param(config.vocab, config.width, dtype=dtype, device=device)
        self.layers = nn.ModuleList([HybridLayer(config, i, dtype, device) for i in range(len(config.layers))])
        self.final_norm = _param(config.width, device=device)
        self.head = _param(config.vocab, config.width, dtype=dtype, device=device)
        self._step_ok: Dict[int, bool] = {}

    # ---- what the registry, the loader and the engine ask of a model
    def tensors(self) -> Dict[str, Tensor]:
        """Checkpoint name -> the (view of the) parameter it fills."""
        out = {"embed": self.embed, "final.norm": self.final_norm, "head": self.head}
        for layer in self.layers:
            out.update(layer.tensors())
        return out

    @property
    def vocab_size(self) -> int:
        return self.config.vocab

    @property
    def window(self) -> int:
        """How many positions back any layer still reads keys (1: none does)."""
        from .mixers import WindowAttention as W
        return max([m.spec.window for l in self.layers for m in l.mixer.mixers if isinstance(m, W)] or [1])

    def new_sequence_state(self, n_slots: int, n_pages: int, page: int, capacity: int) -> List[Any]:
        return [l.mixer.new_state(n_slots, n_pages, page, capacity, self.dtype, self.embed.device) for l in self.layers]

    def step_ok(self, rows: int) -> bool:
        """Whether one-token steps of this many sequences take the fused kernels (which a HIP graph can hold: they
        read positions, slots and pages from device memory and call no library)."""
        if rows not in self._step_ok:
            self._step_ok[rows] = all(l.step_ok(rows) for l in self.layers) and \
                seq_ops.gemv_ok(rows, self.head)
        return self._step_ok[rows]

    def advance(self, ids: Tensor, b: Batch, state: List[Any], starts: Sequence[int], want: Optional[Sequence[int]] = None) -> Tensor:
        return self(ids, b, state, want)

    def forward(self, ids: Tensor, b: Batch, state: List[Any], want: Optional[Sequence[int]] = None,
                layer_outputs: Optional[List[Tensor]] = None) -> Tensor:
        """``ids [B, S]``; returns fp32 logits of the rows ``want`` (row = sequence * S + token; all of them if None).
        ``layer_outputs``: a list that receives the residual stream after every layer."""
        c = self.config
        x = seq_ops.embed(ids, self.embed)
        if b.S == 1 and self.step_ok(b.B):
            for layer, st in zip(self.layers, state):
                layer.step(x, b, st)
                if layer_outputs is not None:
                    layer_outputs.append(x.clone())
            if want is not None and list(want) != list(range(b.B)):
                x = x[list(want)].contiguous()
            if not x.shape[0]:
                return torch.empty((0, c.vocab), dtype=torch.float32, device=x.device)
            return seq_ops.norm_gemv_f32(x, self.final_norm, c.norm_eps, self.head)
        y = None
        for layer, st in zip(self.layers, state):
            y = layer.prompt(x, y, b, st, self.dtype)
            if layer_outputs is not None:
                layer_outputs.append(x + c.residual_mult * y.float())
        if want is not None:
            if not len(want):
                return torch.empty((0, c.vocab), dtype=torch.float32, device=x.device)
            if list(want) != list(range(x.shape[0])):
                rows = torch.tensor(list(want), device=x.device)
                x, y = x[rows], y[rows]
        if seq_ops.gemv_ok(x.shape[0], self.head):
            seq_ops.add_rmsnorm(x, y, c.residual_mult, None, c.norm_eps, self.dtype, norm=False)
            return seq_ops.norm_gemv_f32(x, self.final_norm, c.norm_eps, self.head)
        h = seq_ops.add_rmsnorm(x, y, c.residual_mult, self.final_norm, c.norm_eps, self.dtype)
        return F.linear(h, self.head).float()
