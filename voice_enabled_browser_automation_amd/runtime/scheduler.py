"""Token-level continuous batching over LLMEngine: prompts of token ids in, generated token ids out.

The intent engine (brain/intent_engine.py) schedules grammar-constrained JSON decoding; this is the
plain scheduler for every model of the framework.  An iteration is ONE engine step: each decoding
request contributes its last sampled token, requests still in their prompt a portion of it (as much as
the iteration's token budget leaves), and all rows run together (LLMEngine.step_batch); requests whose
prompt is complete are sampled in one launch.  A request is admitted when a sequence slot is free and the
pool has the blocks its prompt and its longest answer need, so a running request is never starved.
"""
from __future__ import annotations

from collections import deque
from dataclasses import dataclass, field
from typing import Deque, List, Optional, Sequence

import torch

from .engine import LLMEngine, Sequence_


@dataclass
class TokenRequest:
    prompt: List[int]
    max_new: int
    stop_ids: tuple = ()
    out: List[int] = field(default_factory=list)
    feed: List[int] = field(default_factory=list)   # tokens to run before the next sample
    seq: Optional[Sequence_] = None
    reserved: int = 0
    done: bool = False


class TokenScheduler:
    def __init__(self, engine: LLMEngine, *, temperature: float = 0.0, seed: int = 0, token_budget: int = 2048,
                 use_prefix_cache: bool = True):
        self.engine = engine
        self.token_budget = token_budget
        self.use_prefix_cache = use_prefix_cache
        R, dev = engine.max_seqs, engine.device
        self.d_temp = torch.full((R,), float(temperature), dtype=torch.float32, device=dev) if temperature > 0 else None
        self.d_seed = torch.tensor([seed], dtype=torch.int64, device=dev)
        self.d_step = torch.zeros(1, dtype=torch.int32, device=dev)
        self.d_tok = torch.zeros(R, dtype=torch.int32, device=dev)
        self.waiting: Deque[TokenRequest] = deque()
        self.active: List[TokenRequest] = []
        self.stats = dict(iterations=0, rows=0, sampled=0)

    def submit(self, prompt: Sequence[int], max_new: int, stop_ids: Sequence[int] = ()) -> TokenRequest:
        prompt = [int(t) for t in prompt]
        if not prompt or max_new < 1:
            raise ValueError("a request needs a prompt of at least one token and max_new >= 1")
        if len(prompt) + max_new > self.engine.max_model_len:
            raise ValueError(f"prompt + max_new exceed max_model_len={self.engine.max_model_len}")
        if self._blocks(len(prompt) + max_new) > self.engine.blocks.num_blocks - 1:
            raise ValueError("the cache pool is too small for this request")
        r = TokenRequest(prompt=prompt, max_new=max_new, stop_ids=tuple(stop_ids))
        self.waiting.append(r)
        return r

    def _blocks(self, tokens: int) -> int:
        return -(-tokens // self.engine.block_size)

    def _admit(self) -> None:
        eng = self.engine
        while self.waiting and eng.free_sids:
            r = self.waiting[0]
            need = self._blocks(len(r.prompt) + r.max_new)
            held = sum(a.reserved - len(a.seq.blocks) for a in self.active)  # promised, not allocated yet
            if need > eng.blocks.n_free() - held:
                break
            self.waiting.popleft()
            r.seq = eng.new_sequence(r.prompt, use_prefix_cache=self.use_prefix_cache)
            r.reserved = need
            r.feed = r.prompt[r.seq.n_computed:]
            self.active.append(r)

    def has_work(self) -> bool:
        return bool(self.waiting or self.active)

    def step(self) -> List[TokenRequest]:
        """One iteration; returns the requests that finished in it."""
        self._admit()
        entries, sampled, want, n, budget = [], [], [], 0, self.token_budget
        # (decoding requests first: one row each, whatever prompts are in progress)
        for r in sorted(self.active, key=lambda r: not r.out):
            take = r.feed[:budget]
            if not take:
                continue
            entries.append((r.seq, take))
            n += len(take)
            budget -= len(take)
            r.feed = r.feed[len(take):]
            if not r.feed:
                sampled.append(r)
                want.append(n - 1)
        if not entries:
            return []
        logits = self.engine.step_batch(entries, want)
        self.stats["iterations"] += 1
        self.stats["rows"] += n
        if not sampled:
            return []
        k = len(sampled)
        self.engine.sample(logits, mask=None, temperature=None if self.d_temp is None else self.d_temp[:k],
                           seed=self.d_seed, step=self.d_step, out_tokens=self.d_tok[:k])
        toks = self.d_tok[:k].tolist()
        self.engine.host_synced()
        self.stats["sampled"] += k
        finished = []
        for r, t in zip(sampled, toks):
            if t < 0:
                raise RuntimeError(f"no finite logit to sample from (code {t})")
            r.out.append(t)
            if t in r.stop_ids or len(r.out) >= r.max_new:
                r.done = True
                self.engine.free_sequence(r.seq)
                finished.append(r)
            else:
                r.feed = [t]
        if finished:
            self.active = [r for r in self.active if not r.done]
        return finished

    def run_until_idle(self) -> None:
        while self.has_work():
            self.step()

    def generate(self, prompts: Sequence[Sequence[int]], max_new: int, stop_ids: Sequence[int] = ()) -> List[List[int]]:
        reqs = [self.submit(p, max_new, stop_ids) for p in prompts]
        while not all(r.done for r in reqs):
            self.step()
        return [r.out for r in reqs]
