"""Continuous batching for LocalEngine: requests of any length share steps.

Every step runs one token of each request that is decoding beside portions of
the prompts that are not finished, up to a token budget, as one ragged batch
(kv/batch.py). A request is admitted when the KV pool can promise its whole
length, and gives its pages back as soon as it ends, so the next one in line
starts in the middle of the others' generation. Steps in which everyone decodes
replay the engine's captured graph.
"""
from __future__ import annotations

from collections import deque
from dataclasses import dataclass, field
from typing import Deque, List, Optional, Sequence

import torch

from bloombee_amd.client.generation import RemoteGenerationMixin
from bloombee_amd.kv.paged import AllocationFailed, SessionHandle


@dataclass
class Request:
    prompt: List[int]
    max_new_tokens: int
    do_sample: bool = False
    temperature: float = 1.0
    top_k: Optional[int] = None
    top_p: Optional[float] = None
    generator: Optional[torch.Generator] = None
    eos_token_id: Optional[int] = None
    output: List[int] = field(default_factory=list)
    fed: int = 0                      # prompt tokens already run
    handle: Optional[SessionHandle] = None
    done: bool = False


class BatchScheduler:
    def __init__(self, engine, max_batch: int = 32, chunk_tokens: int = 2048):
        if max_batch < 1 or chunk_tokens < 1:
            raise ValueError("max_batch and chunk_tokens must be positive")
        self.engine = engine
        self.max_batch = max_batch
        self.chunk_tokens = chunk_tokens    # tokens of one step, at most
        self.waiting: Deque[Request] = deque()
        self.running: List[Request] = []

    def submit(self, prompt: Sequence[int], max_new_tokens: int,
               **sampling) -> Request:
        req = Request(list(prompt), max_new_tokens, **sampling)
        total = len(req.prompt) + max_new_tokens
        cap = min(self.engine.config.max_position_embeddings,
                  self.engine.kv_pool.max_tokens)
        if not req.prompt or max_new_tokens < 1:
            raise ValueError("a request needs a prompt and a token to make")
        if total - 1 > cap:      # the last token is never fed back
            raise ValueError(f"request of {total} tokens exceeds {cap}")
        self.waiting.append(req)
        return req

    def _admit(self) -> None:
        while self.waiting and len(self.running) < self.max_batch:
            req = self.waiting[0]
            length = len(req.prompt) + req.max_new_tokens - 1
            try:
                req.handle = self.engine.kv_pool.allocate(1, length, timeout=0)
            except AllocationFailed:
                if not self.running:
                    raise     # nobody left to give pages back
                return
            self.running.append(self.waiting.popleft())

    def step(self) -> bool:
        """Run one mixed step; False once nothing is left to do."""
        self._admit()
        if not self.running:
            return False
        decoding = [r for r in self.running if r.output]
        filling = [r for r in self.running if not r.output]
        if not filling:
            logits = self.engine.decode([(r.handle, r.output[-1])
                                         for r in decoding])
            self._take(decoding, logits)
            return True
        budget = max(1, self.chunk_tokens - len(decoding))
        entries = [(r.handle, [r.output[-1]], [0]) for r in decoding]
        ready = list(decoding)
        for r in filling:
            n = min(budget, len(r.prompt) - r.fed)
            if n < 1:
                break
            part = r.prompt[r.fed:r.fed + n]
            r.fed += n
            budget -= n
            last = r.fed == len(r.prompt)
            entries.append((r.handle, part, [n - 1] if last else []))
            if last:
                ready.append(r)
        logits = self.engine.step(entries)
        self._take(ready, logits)
        return True

    def _take(self, reqs: List[Request], logits: torch.Tensor) -> None:
        if not reqs:
            return
        greedy = None
        for i, r in enumerate(reqs):
            if r.do_sample:
                tok = int(RemoteGenerationMixin._pick(
                    logits[i:i + 1], True, r.temperature, r.top_k, r.top_p,
                    r.generator))
            else:
                if greedy is None:
                    greedy = logits.argmax(-1).tolist()
                tok = greedy[i]
            r.output.append(tok)
            if len(r.output) >= r.max_new_tokens or tok == r.eos_token_id:
                r.done = True
                r.handle.close()
        self.running = [r for r in self.running if not r.done]

    def run(self) -> None:
        while self.step():
            pass
