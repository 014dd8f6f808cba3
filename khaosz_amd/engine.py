"""Running a registered model over sequences: one step function on the cache, and generation on top of it.

``step`` feeds the next tokens of some sequences and returns logits; ``generate`` schedules prompts and decoding over
it (a prompt is run in portions, running sequences decode together, as astrai/inference/core/scheduler.py:119-196
groups them).  One-token steps of a model whose kernels read their positions from device memory are captured in a HIP
graph, one per batch size, and replayed for every later step.
"""
from __future__ import annotations

from typing import Dict, Iterable, List, NamedTuple, Optional, Sequence

import numpy as np
import torch
from torch import Tensor

from .cache import SequenceCache
from .sampling import Sampler

MAX_DECODE_BATCH = 8
PROMPT_PORTION = 4096


class _Captured(NamedTuple):
    graph: torch.cuda.CUDAGraph
    words: Tensor   # device, what the graph reads
    host: Tensor    # pinned
    logits: Tensor


class Engine:
    def __init__(self, model, max_tokens: int, max_seqs: int = 1, page: int = 64, graphs: bool = True):
        self.model = model
        self.device = next(model.parameters()).device
        self.cache = SequenceCache(model, max_tokens, max_seqs, page)
        self.max_seqs = max_seqs
        self._use_graphs = graphs and self.device.type == "cuda"
        self._graphs: Dict[int, _Captured] = {}
        self._warm: set = set()

    # ---- sequences
    def open(self) -> int:
        return self.cache.open()

    def close(self, handle: int) -> None:
        self.cache.close(handle)

    @torch.inference_mode()
    def step(self, handles: Sequence[int], tokens: Sequence[Sequence[int]], want: Optional[Sequence[int]] = None) -> Tensor:
        """The next ``tokens[i]`` of sequence ``handles[i]`` (equally many for each).  Returns fp32 logits of the rows
        ``want`` (row = i * S + token; all if None); the tensor is valid until the next step."""
        B, S = len(handles), len(tokens[0])
        if B == 0 or S == 0 or any(len(t) != S for t in tokens) or len(set(handles)) != B:
            raise ValueError("a step takes equally many new tokens, at least one, of distinct sequences")
        ids = np.asarray(tokens, np.int64)
        if ids.min() < 0 or ids.max() >= self.model.vocab_size:
            raise ValueError("token id outside the vocabulary")
        if want is not None and any(not 0 <= w < B * S for w in want):
            raise ValueError("a wanted row is not among the tokens of this step")
        self.cache.reserve(handles, S)
        if S == 1 and self._use_graphs and self.model.step_ok(B):
            logits = self._graph_step(handles, ids)
            if want is not None and list(want) != list(range(B)):
                logits = logits[list(want)]
        else:
            logits = self._eager(handles, ids, want)
        self.cache.commit(handles, S)
        return logits

    def _eager(self, handles, ids, want) -> Tensor:
        B, S = ids.shape
        words = np.empty(self.cache.words(B, S), np.int64)
        self.cache.pack(handles, ids, words)
        dev_ids, batch = self.cache.unpack(torch.from_numpy(words).to(self.device), B, S)
        return self.model.advance(dev_ids, batch, self.cache.state, [self.cache.length(h) for h in handles], want)

    def _graph_step(self, handles, ids) -> Tensor:
        B = len(handles)
        if B not in self._warm:  # the first step of a size runs as it is: it loads what a capture must not load
            self._warm.add(B)
            return self._eager(handles, ids, None)
        c = self._graphs.get(B)
        if c is None:
            c = self._graphs[B] = self._capture(B)
        torch.cuda.current_stream(self.device).synchronize()  # the previous copy out of the pinned words is done
        self.cache.pack(handles, ids, c.host.numpy())
        c.words.copy_(c.host, non_blocking=True)
        c.graph.replay()
        return c.logits

    def _capture(self, B: int) -> _Captured:
        n = self.cache.words(B, 1)
        words = torch.zeros(n, dtype=torch.int64, device=self.device)
        host = torch.zeros(n, dtype=torch.int64, pin_memory=True)
        dev_ids, batch = self.cache.unpack(words, B, 1)
        graph = torch.cuda.CUDAGraph()
        with torch.cuda.graph(graph):
            logits = self.model.advance(dev_ids, batch, self.cache.state, [0] * B, None)
        return _Captured(graph, words, host, logits)

    # ---- generation
    def prefill(self, handle: int, tokens: Sequence[int]) -> Tensor:
        """A whole prompt in portions; the logits of its last token ``[1, vocab]``."""
        for at in range(0, len(tokens), PROMPT_PORTION):
            part = tokens[at:at + PROMPT_PORTION]
            last = at + len(part) == len(tokens)
            logits = self.step([handle], [part], [len(part) - 1] if last else [])
        return logits

    def generate(self, prompts: Sequence[Sequence[int]], max_new_tokens: int, sampler: Optional[Sampler] = None,
                 stop: Iterable[int] = ()) -> List[List[int]]:
        """Continuations of ``prompts``; a sequence ends after ``max_new_tokens`` or with a token of ``stop``."""
        sampler, stop = sampler or Sampler(), set(stop)
        out: List[List[int]] = [[] for _ in prompts]
        waiting = [i for i, p in enumerate(prompts) if max_new_tokens > 0]
        running: Dict[int, int] = {}  # prompt -> handle

        def done(i: int) -> bool:
            return len(out[i]) >= max_new_tokens or (bool(out[i]) and out[i][-1] in stop)

        try:
            while waiting or running:
                while waiting and len(running) < self.max_seqs and self._fits(prompts, waiting[0], running, max_new_tokens):
                    i = waiting.pop(0)
                    running[i] = self.open()
                    out[i].append(int(sampler(self.prefill(running[i], list(prompts[i])))[0]))
                    if done(i):
                        self.close(running.pop(i))
                if not running:
                    continue
                group = self._group(running)
                logits = self.step([running[i] for i in group], [[out[i][-1]] for i in group])
                for i, t in zip(group, sampler(logits).tolist()):
                    out[i].append(int(t))
                    if done(i):
                        self.close(running.pop(i))
        finally:
            for h in running.values():
                self.close(h)
        return out

    def _fits(self, prompts, i: int, running: Dict[int, int], new: int) -> bool:
        """Whether every running sequence and this one can reach their full length."""
        pages = lambda n: (n + self.cache.page - 1) // self.cache.page
        need = [pages(len(prompts[k]) + new) for k in list(running) + [i]]
        if need[-1] > self.cache.width or not prompts[i]:
            raise ValueError(f"prompt {i} with {new} new tokens does not fit the cache (or is empty)")
        return sum(need) <= self.cache.width + self.max_seqs - 1

    def _group(self, running: Dict[int, int]) -> List[int]:
        """The sequences of the next decode step: all of them, or the largest group at one position where the model
        asks for that."""
        items = sorted(running)
        if not self.model.mixed_positions:
            by_pos: Dict[int, List[int]] = {}
            for i in items:
                by_pos.setdefault(self.cache.length(running[i]), []).append(i)
            items = max(by_pos.values(), key=len)
        # those that are furthest behind first, so that a batch that does not hold all starves none
        return sorted(items, key=lambda i: self.cache.length(running[i]))[:MAX_DECODE_BATCH]
