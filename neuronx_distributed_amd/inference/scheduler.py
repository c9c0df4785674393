"""Continuous batching on the serving engine.

Every iteration packs one token of each decoding request and portions of
waiting prompts, up to a token budget, into one engine step.  A request is
admitted when a slot is free and the pages of its prompt and its whole
output are, so a running request is never pushed out.
"""

from collections import deque
from dataclasses import dataclass, field
from typing import Dict, List, Optional, Sequence

from ..utils.sampling import Sampler
from .engine import InferenceEngine, StepEntry
from .paged_cache import PAGE_SIZE, CacheManager


@dataclass
class Request:
    id: int
    prompt: List[int]
    max_new_tokens: int
    eos_token_id: int = -1
    done_prompt: int = 0
    output: List[int] = field(default_factory=list)

    @property
    def finished(self) -> bool:
        return len(self.output) >= self.max_new_tokens or (
            self.eos_token_id >= 0 and bool(self.output)
            and self.output[-1] == self.eos_token_id)


class Scheduler:
    def __init__(self, engine: InferenceEngine,
                 sampler: Optional[Sampler] = None,
                 max_step_tokens: int = 2048,
                 max_portion: Optional[int] = None):
        self.engine = engine
        self.sampler = sampler or Sampler(do_sample=False)
        self.max_step_tokens = max(1, max_step_tokens)
        self.max_portion = max_portion or self.max_step_tokens
        self.waiting: deque = deque()
        self.running: Dict[int, Request] = {}
        self._reserved = 0
        self._next_id = 0

    def submit(self, prompt: Sequence[int], max_new_tokens: int,
               eos_token_id: int = -1) -> Request:
        if not len(prompt):
            raise ValueError("a prompt needs at least one token")
        r = Request(self._next_id, [int(t) for t in prompt],
                    int(max_new_tokens), eos_token_id)
        if r.max_new_tokens < 1:
            return r
        c = self.engine.cache
        total = len(r.prompt) + r.max_new_tokens
        if total > c.max_context or (c.paged and self._pages(r) >
                                     c.num_pages):
            raise ValueError(f"a request of {total} tokens does not fit the "
                             "cache")
        self._next_id += 1
        self.waiting.append(r)
        return r

    def _pages(self, r: Request) -> int:
        c = self.engine.cache
        return c.pages_for(len(r.prompt) + r.max_new_tokens) if c.paged else 0

    def _admit(self):
        c = self.engine.cache
        while self.waiting and len(self.running) < c.num_slots:
            need = self._pages(self.waiting[0])
            if self._reserved + need > c.num_pages:
                return
            r = self.waiting.popleft()
            self._reserved += need
            self.running[r.id] = r

    def step(self) -> List[Request]:
        """One engine step; returns the requests that finished with it."""
        self._admit()
        entries, budget = [], self.max_step_tokens
        for r in self.running.values():     # decoding requests first
            if r.done_prompt == len(r.prompt) and budget > 0:
                entries.append(StepEntry(r.id, [r.output[-1]], [0]))
                budget -= 1
        for r in self.running.values():
            left = len(r.prompt) - r.done_prompt
            n = min(left, budget, self.max_portion)
            if n <= 0:
                continue
            part = r.prompt[r.done_prompt:r.done_prompt + n]
            r.done_prompt += n
            budget -= n
            entries.append(StepEntry(r.id, part,
                                     [n - 1] if n == left else []))
        if not entries:
            return []
        logits = self.engine.step(entries)
        ended = []
        if logits is not None:
            toks = self.sampler(logits).tolist()
            for e, t in zip([e for e in entries if e.want], toks):
                r = self.running[e.id]
                r.output.append(int(t))
                if r.finished:
                    ended.append(r)
        for r in ended:
            self.engine.finish(r.id)
            self._reserved -= self._pages(r)
            del self.running[r.id]
        return ended

    def run(self) -> List[Request]:
        """Step until nothing waits or runs."""
        out = []
        while self.waiting or self.running:
            out += self.step()
        return out


def generate_ragged(model, prompts: Sequence[Sequence[int]],
                    max_new_tokens: int = 32,
                    sampler: Optional[Sampler] = None, eos_token_id: int = -1,
                    max_seqs: Optional[int] = None,
                    max_step_tokens: int = 2048,
                    use_graphs: bool = True) -> List[List[int]]:
    """Generate for prompts of unequal length; returns the new tokens of
    each, in order."""
    if not prompts:
        return []
    max_seqs = max_seqs or min(len(prompts), 64)
    per = sorted((CacheManager.pages_for(len(p) + max_new_tokens) * PAGE_SIZE
                  for p in prompts), reverse=True)
    engine = InferenceEngine(model, max_tokens=sum(per[:max_seqs]),
                             max_seqs=max_seqs, max_context=per[0],
                             use_graphs=use_graphs)
    sched = Scheduler(engine, sampler, max_step_tokens)
    reqs = [sched.submit(p, max_new_tokens, eos_token_id) for p in prompts]
    sched.run()
    return [r.output for r in reqs]
