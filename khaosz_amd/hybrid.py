"""Decoders whose layers mix linear recurrences, windowed and latent attention, configured layer by layer.

Two designs share the layers, the model class and everything behind it:

* ``Rudilix``: pre-norm layers ``x += m mixer(norm(x)); x += m ff(norm(x))`` with mixers of three kinds (``mamba2``,
  ``channel_delta``, and ``parallel``: windowed attention beside a channel delta rule), norms with their weight around zero,
  clamped GLU feed-forwards.
* ``Lomozen``: norms before and after each sublayer, ``x += norm'(mixer(norm(x))); x += norm'(ff(norm(x)))``, with mixers of two
  kinds (``latent_attention``, ``lightning``), plain norm weights, routed experts with a shared one.

Both have an untied vocabulary projection.  Which mixer a layer has, every size and every constant that is not the design's
come from the configuration.  The residual stream is fp32 throughout; weights and activations are bf16 or fp32.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Callable, Dict, List, NamedTuple, Optional, Sequence

import torch
import torch.nn as nn
import torch.nn.functional as F
from torch import Tensor

from . import seq_ops
from .mixers import (Branch, ChannelDeltaMixer, ClampedGLU, LatentAttention, LightningMixer, Mamba2Mixer, MixerBlock, RoutedExperts,
                     WindowAttention, _param)
from .registry import register_model
from .seq_ops import Batch, Stream


class Design(NamedTuple):
    """What a design fixes: the mixers a layer's ``type`` may name, the feed-forwards its ``kind`` may name, what is added to
    a norm's stored weight, and whether a sublayer's output passes a norm of its own."""
    mixers: Dict[str, Callable]
    feed_forwards: Dict[str, Callable]
    norm_offset: float
    post_norms: bool


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
    architecture: str = "Rudilix"

    @property
    def design(self) -> Design:
        return DESIGNS[self.architecture]

    @classmethod
    def from_dict(cls, d: Dict[str, Any], shapes: Optional[Dict[str, Sequence[int]]] = None) -> "HybridConfig":
        name = d.get("architecture", "Rudilix")
        if name not in DESIGNS:
            raise ValueError(f"unknown design {name!r}, know {sorted(DESIGNS)}")
        design = DESIGNS[name]
        for i, layer in enumerate(d["layers"]):
            if layer["type"] not in design.mixers:
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}, know {sorted(design.mixers)}")
            mlp = layer.get("mlp")
            if mlp is not None and mlp["kind"] not in design.feed_forwards:
                raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
        ranks = {n: s[0] for n, s in (shapes or {}).items() if n.endswith((".a1", ".g1"))}
        return cls(int(d["vocab"]), int(d["width"]), d["layers"], float(d["norm"]["eps"]), float(d.get("residual_mult", 1.0)), ranks, name)


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


def _alone(mixer) -> Callable:
    return lambda cfg, c, prefix, dtype, device: [("", mixer(c, cfg.norm_eps, dtype, device), 1.0)]


DESIGNS = {
    "Rudilix": Design({"mamba2": _alone(Mamba2Mixer), "channel_delta": _delta, "parallel": _parallel}, {"dense": ClampedGLU}, 1.0, False),
    "Lomozen": Design({"latent_attention": _alone(LatentAttention), "lightning": _alone(LightningMixer)}, {"moe": RoutedExperts}, 0.0, True),
}


class HybridLayer(nn.Module):
    def __init__(self, cfg: HybridConfig, index: int, dtype, device=None):
        super().__init__()
        layer, design = cfg.layers[index], cfg.design
        self.prefix, self.eps, self.mult, self.w0 = f"l{index}.", cfg.norm_eps, cfg.residual_mult, design.norm_offset
        mixers = design.mixers[layer["type"]](cfg, layer["mixer"], self.prefix + "mix.", dtype, device)
        norm = lambda on: _param(cfg.width, device=device) if on else None
        self.norm1, self.norm1b = norm(True), norm(design.post_norms)
        self.mixer = MixerBlock(cfg.width, mixers, dtype, device)
        mlp = layer.get("mlp")
        self.norm2, self.norm2b = norm(mlp is not None), norm(mlp is not None and design.post_norms)
        self.mlp = design.feed_forwards[mlp["kind"]](cfg.width, mlp, dtype, device) if mlp is not None else None

    def tensors(self) -> Dict[str, Tensor]:
        norms = lambda *names: {self.prefix + n: t for n in names if (t := getattr(self, n)) is not None}
        out = norms("norm1", "norm1b")
        out.update({self.prefix + "mix." + n: t for n, t in self.mixer.tensors().items()})
        out.update(norms("norm2", "norm2b"))
        if self.mlp is not None:
            out.update({self.prefix + "mlp." + n: t for n, t in self.mlp.tensors().items()})
        return out

    def _norm(self, x: Tensor, pending: Optional[Branch], w: Tensor, dtype) -> Tensor:
        return add_branch(x, pending, self.mult, w, self.eps, dtype, self.w0)

    def prompt(self, x: Tensor, pending: Optional[Branch], b: Batch, st, dtype) -> Branch:
        """Adds the pending branch output to the stream, runs the layer and returns its own pending output."""
        y = self.mixer.prompt(self._norm(x, pending, self.norm1, dtype), b, st)._replace(post=self.norm1b)
        if self.mlp is None:
            return y
        return self.mlp.prompt(self._norm(x, y, self.norm2, dtype))._replace(post=self.norm2b)

    def step(self, s: Stream, b: Batch, st) -> None:
        self.mixer.step(s, self.norm1, b, st, self.norm1b)
        if self.mlp is not None:
            self.mlp.step(s, self.norm2, self.norm2b)

    def step_ok(self, rows: int) -> bool:
        return self.mixer.step_ok(rows) and (self.mlp is None or self.mlp.step_ok(rows))


def add_branch(x: Tensor, pending: Optional[Branch], mult: float, w: Optional[Tensor], eps: float, dtype, w0: float) -> Optional[Tensor]:
    """Adds a pending branch output to the stream ``x`` in place; returns the sum normed with ``w0 + w`` if there is a ``w``."""
    p = pending or Branch(None)
    return seq_ops.add_rmsnorm(x, p.y, mult, w, eps, dtype, w is not None, w0, p.post, p.routed)


@register_model("Rudilix")
@register_model("Lomozen")
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
        return max([m.spec.window for l in self.layers for m in l.mixer.mixers if isinstance(m, (WindowAttention, LatentAttention))] or [1])

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
        return self(ids, b._replace(starts=tuple(starts)) if b.S > 1 or not self.step_ok(b.B) else b, state, want)

    def forward(self, ids: Tensor, b: Batch, state: List[Any], want: Optional[Sequence[int]] = None,
                layer_outputs: Optional[List[Tensor]] = None) -> Tensor:
        """``ids [B, S]``; returns fp32 logits of the rows ``want`` (row = sequence * S + token; all of them if None).
        ``layer_outputs``: a list that receives the residual stream after every layer."""
        c, w0 = self.config, self.config.design.norm_offset
        x = seq_ops.embed(ids, self.embed)
        if b.S == 1 and self.step_ok(b.B):
            s = Stream(x, c.norm_eps, w0, c.residual_mult)
            for layer, st in zip(self.layers, state):
                layer.step(s, b, st)
                if layer_outputs is not None:
                    layer_outputs.append(s.settled())
            if want is not None and list(want) != list(range(b.B)):
                s.rows(list(want))
            if not s.x.shape[0]:
                return torch.empty((0, c.vocab), dtype=torch.float32, device=x.device)
            return s.norm_gemv_f32(self.final_norm, self.head)
        pending = None
        for layer, st in zip(self.layers, state):
            pending = layer.prompt(x, pending, b, st, self.dtype)
            if layer_outputs is not None:
                layer_outputs.append(x.clone())
                add_branch(layer_outputs[-1], pending, c.residual_mult, None, c.norm_eps, self.dtype, w0)
        if want is not None:
            if not len(want):
                return torch.empty((0, c.vocab), dtype=torch.float32, device=x.device)
            if list(want) != list(range(x.shape[0])):
                rows = torch.tensor(list(want), device=x.device)
                x, pending = x[rows], pending.rows(rows)
        if seq_ops.gemv_ok(x.shape[0], self.head):
            add_branch(x, pending, c.residual_mult, None, c.norm_eps, self.dtype, w0)
            return Stream(x, c.norm_eps, w0, c.residual_mult).norm_gemv_f32(self.final_norm, self.head)
        return F.linear(add_branch(x, pending, c.residual_mult, self.final_norm, c.norm_eps, self.dtype, w0), self.head).float()
