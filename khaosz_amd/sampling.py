"""Choosing the next token from logits: greedy, or temperature, top-k and nucleus filtering and one draw
(the pipeline of astrai/inference/sample.py:34-190)."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch
from torch import Tensor


@dataclass
class Sampler:
    temperature: float = 0.0  # 0: greedy
    top_k: int = 0            # 0: off
    top_p: float = 1.0        # 1: off
    seed: Optional[int] = None

    def __post_init__(self):
        if self.temperature < 0 or self.top_k < 0 or not 0 < self.top_p <= 1:
            raise ValueError("temperature and top_k must not be negative, top_p in (0, 1]")
        self._generators = {}

    def __call__(self, logits: Tensor) -> Tensor:
        """``logits [n, vocab]`` -> token ids ``[n]``."""
        if self.temperature == 0:
            return logits.argmax(-1)
        z = logits.float() / self.temperature
        if 0 < self.top_k < z.shape[-1]:
            z = z.masked_fill(z < z.topk(self.top_k, dim=-1).values[:, -1:], float("-inf"))
        if self.top_p < 1:
            order = z.sort(dim=-1, descending=True)
            p = order.values.softmax(-1)
            drop = (p.cumsum(-1) - p) >= self.top_p  # the mass in front of a token is enough already
            z = z.masked_fill(torch.zeros_like(drop).scatter(-1, order.indices, drop), float("-inf"))
        g = self._generators.get(z.device)
        if g is None:
            g = self._generators[z.device] = torch.Generator(device=z.device)
            g.manual_seed(self.seed) if self.seed is not None else g.seed()
        return torch.multinomial(z.softmax(-1), 1, generator=g)[:, 0]
