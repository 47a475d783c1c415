"""Batched serving of the layered designs: requests of different lengths in one step, over one paged cache.

`BatchEngine.step` takes the next tokens of any number of requests and returns the logits asked for: single tokens of running
requests go through the decode step, anything else (new prompts, portions of prompts, a mixture) through the ragged prompt pass.
`generate_batch` is the scheduler on top: it admits requests, prefills them (in portions when asked), decodes the running batch
token by token with the framework's sampler and retires each request at its own length.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, Hashable, List, Optional, Sequence

import numpy as np
import torch

from .. import runtime
from ..kernels import layered as K
from .layered import GraphedPrompt, LayeredTransformer, PromptBatch, StepBatch
from .layered_engine import LayeredEngine


class BatchEngine:
    """max_tokens: tokens the live requests are expected to hold together (the cache grows past it); graphs: replay decode steps (per
    batch size) and short prompts (per shape of the batch) from hipGraphs, captured at their second use."""

    MAX_GRAPHS = 16

    def __init__(self, model: LayeredTransformer, max_tokens: int = 4096, max_requests: int = 8, graphs: bool = False):
        self.model = model
        self.device = model.tok_embeddings.weight.device
        self.cache = model.new_cache(max_tokens, max_requests)
        self.slot: Dict[Hashable, int] = {}
        self.graphs = graphs
        # one running request, 16-bit: the fused step (same cache, same attention kernels)
        self.fused = LayeredEngine(model, cache=self.cache, max_seq=8) if LayeredEngine.supports(model, need_caches=False) is None else None
        self.prompt = GraphedPrompt(model) if graphs else model.prompt_pass
        self._graphs: Dict[tuple, tuple] = {}
        self._seen: set = set()

    def _decode(self, dev: torch.Tensor, max_pos: int, hook=None) -> torch.Tensor:
        """one step of the tokens dev[0] at positions dev[1] of slots dev[2]"""
        if dev.shape[1] == 1 and self.fused is not None and hook is None:
            self.fused.max_pos = max_pos
            self.fused.slot = dev[2]
            return self.fused(dev[0], dev[1]).view(1, -1)
        return self.model.step_pass(StepBatch(self.cache, dev[0], dev[1], dev[2], max_pos), hook)

    def _decode_graphed(self, flat: np.ndarray) -> torch.Tensor:
        # (the positions only choose how far the attention is split: a power of two, so that a graph serves many steps)
        max_pos = max(256, 1 << int(flat[1].max()).bit_length()) - 1
        key = (flat.shape[1], max_pos, self.cache.version)
        if key not in self._graphs:
            dev = torch.from_numpy(flat).to(self.device)
            if key not in self._seen:
                if len(self._seen) >= 1024:
                    self._seen.clear()
                self._seen.add(key)
                return self._decode(dev, max_pos)
            torch.cuda.synchronize()
            for k in [k for k in self._graphs if k[2] != key[2]] + (list(self._graphs)[:1] if len(self._graphs) >= self.MAX_GRAPHS else []):
                self._graphs.pop(k, None)  # a graph over a replaced cache buffer, or the oldest one
            g = torch.cuda.CUDAGraph()
            with runtime.graph_capture(g):
                logits = self._decode(dev, max_pos)
            self._graphs[key] = (g, dev, logits)
        g, dev, logits = self._graphs[key]
        dev.copy_(torch.from_numpy(flat))
        g.replay()
        return logits

    def length(self, rid: Hashable) -> int:
        return self.cache.lengths[self.slot[rid]] if rid in self.slot else 0

    def step(self, entries: Sequence[tuple], hook=None) -> Optional[torch.Tensor]:
        """entries: [(request, its next tokens, places among them whose logits are wanted)].  Returns fp32 [wanted, vocab] in the order
        of the entries and places, or None when nothing is wanted."""
        vocab = self.model.config.vocab_size
        batch, want, at = [], [], 0
        for rid, tokens, places in entries:
            if not len(tokens) or min(tokens) < 0 or max(tokens) >= vocab or any(not 0 <= k < len(tokens) for k in places):
                raise ValueError(f"request {rid!r}: no tokens, a token outside the vocabulary or a place outside the tokens")
        if len({e[0] for e in entries}) != len(entries):
            raise ValueError("a request appears twice in one step")
        for rid, tokens, places in entries:
            if rid not in self.slot:
                self.slot[rid] = self.cache.open()
            s = self.slot[rid]
            start = self.cache.lengths[s]
            self.cache.extend(s, start + len(tokens))
            batch.append((s, start, tokens))
            want.extend(at + k for k in places)
            at += len(tokens)
        self.cache.sync()
        if all(start > 0 and len(t) == 1 for _, start, t in batch):
            flat = np.asarray([[t[0] for _, _, t in batch], [st for _, st, _ in batch], [s for s, _, _ in batch]], dtype=np.int32)
            if self.graphs and hook is None:
                logits = self._decode_graphed(flat)
            else:
                logits = self._decode(torch.from_numpy(flat).to(self.device), int(flat[1].max()), hook)
            # (a copy: the next step overwrites the buffer of the fused step and of a graph)
            out = None if not want else logits.clone() if len(want) == len(batch) else logits[torch.tensor(want, device=self.device)]
        else:
            b = PromptBatch(self.cache, batch, self.device)
            out = self.prompt(b, want) if hook is None else self.model.prompt_pass(b, want, hook)
        for s, _, _ in batch:
            self.cache.trim(s)
        return out

    def release(self, rid: Hashable) -> None:
        """the request is finished: its pages and slot go back"""
        self.cache.close(self.slot.pop(rid))


@dataclass
class Request:
    prompt: Sequence[int]
    max_new_tokens: int


@torch.no_grad()
def generate_batch(model: LayeredTransformer, requests: Sequence[Request], temperature: float = 0.0, top_k: Optional[int] = None,
                   max_batch: int = 64, portion: Optional[int] = None, engine: Optional[BatchEngine] = None, seed: int = 1234,
                   graphs: bool = True) -> List[List[int]]:
    """New tokens of every request.  At most max_batch run at a time, a waiting request is admitted as soon as one retires;
    prompts enter whole or `portion` tokens at a time.  temperature <= 0: greedy; else the framework's top-k sampler."""
    eng = engine or BatchEngine(model, max_tokens=max(sum(len(r.prompt) + r.max_new_tokens for r in requests[:max_batch]), 64), max_requests=max_batch, graphs=graphs)
    # a random stream per request: what a request draws does not depend on what runs next to it
    rng = torch.tensor([[seed + i, 0] for i in range(len(requests))], dtype=torch.int64, device=eng.device)
    out: List[List[int]] = [[] for _ in requests]
    waiting = [i for i, r in enumerate(requests) if r.max_new_tokens > 0]
    running: List[int] = []

    def emit(ids, logits):
        at = torch.tensor(ids, device=eng.device)
        state = rng[at]
        tokens = K.sample_rows(logits, state, temperature, top_k).tolist()
        rng[at] = state
        for i, t in zip(ids, tokens):
            out[i].append(t)
            if len(out[i]) >= requests[i].max_new_tokens:
                eng.release(i)
                if i in running:
                    running.remove(i)
            elif i not in running:
                running.append(i)

    while waiting or running:
        new = [waiting.pop(0) for _ in range(min(len(waiting), max_batch - len(running)))]
        if new:
            size = portion or max(len(requests[i].prompt) for i in new)
            left = {i: list(requests[i].prompt) for i in new}
            while left:
                entries, done = [], []
                for i in list(left):
                    part, left[i] = left[i][:size], left[i][size:]
                    if not left[i]:
                        del left[i]
                        done.append(i)
                    entries.append((i, part, [len(part) - 1] if i in done else []))
                logits = eng.step(entries)
                if done:
                    emit(done, logits)
        if running:
            ids = list(running)
            emit(ids, eng.step([(i, [out[i][-1]], [0]) for i in ids]))
    return out
