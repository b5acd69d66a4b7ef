"""`TokenBatcher` - request scheduler of the token language models: the counterpart of `SessionBatcher` for prompts.

Requests queue, are admitted when a slot and the pages of their whole length are there, and run in mixed batches: every step takes
one token of each decoding request first and fills the rest of its token budget with portions of prompts.

    batcher = TokenBatcher(lm, step_tokens=2048)
    rid = batcher.submit(prompt_ids, max_new_tokens=64)                # temp=0: greedy
    while batcher.step():
        ...
    tokens = batcher.pop(rid)                                          # None until the request has finished

`generate` does the loop for a list of prompts.
"""
from __future__ import annotations

from collections import deque
from dataclasses import dataclass, field
from typing import Deque, Dict, Iterable, List, Optional, Sequence

from .errors import UnknownChannel
from .tlm import TokenLM


@dataclass
class _Request:
    rid: int
    prompt: List[int]
    max_new: int
    temp: float
    top_k: int
    stop: frozenset
    slot: int = -1
    fed: int = 0                         # prompt tokens the engine has seen
    out: List[int] = field(default_factory=list)
    pages: int = 0                       # pages the admission reserved

    @property
    def prefilling(self) -> bool:
        return self.fed < len(self.prompt)


class TokenBatcher:
    def __init__(self, lm: TokenLM, step_tokens: int = 2048, seed: int = 0):
        self.lm = lm
        self.step_tokens = min(int(step_tokens), lm.max_step_tokens)
        if self.step_tokens < 1:
            raise ValueError("step_tokens must be positive")
        self.seed = int(seed)
        self._waiting: Deque[_Request] = deque()
        self._live: List[_Request] = []
        self._done: Dict[int, List[int]] = {}
        self._next = 1
        self._reserved = 0               # pages live requests were promised

    # ---- requests --------------------------------------------------------------------------------------------------
    def submit(self, prompt: Sequence[int], max_new_tokens: int, temp: float = 0.0, top_k: int = 0, stop: Iterable[int] = ()) -> int:
        prompt = [int(t) for t in prompt]
        if not prompt or max_new_tokens < 1:
            raise ValueError("a request needs a prompt and at least one new token")
        if any(t < 0 or t >= self.lm.vocab for t in prompt):
            raise ValueError("token outside the vocabulary")
        limit = getattr(self.lm, "max_positions", 0)
        if limit and len(prompt) + max_new_tokens - 1 > limit:
            raise ValueError(f"the request reaches position {len(prompt) + max_new_tokens - 1}, the model has {limit}")
        need = self.lm.pages_needed(-1, len(prompt) + max_new_tokens - 1)
        if need > self.lm.total_pages:
            raise BufferError(f"the request needs {need} pages, the pool has {self.lm.total_pages}")
        r = _Request(self._next, prompt, int(max_new_tokens), float(temp), int(top_k), frozenset(int(t) for t in stop), pages=need)
        self._next += 1
        self._waiting.append(r)
        return r.rid

    def cancel(self, rid: int) -> None:
        for r in list(self._live):
            if r.rid == rid:
                self._finish(r, keep=False)
                return
        for r in list(self._waiting):
            if r.rid == rid:
                self._waiting.remove(r)
                return
        if self._done.pop(rid, None) is None:
            raise UnknownChannel(f"no request {rid}")

    def pop(self, rid: int) -> Optional[List[int]]:
        """The finished request's tokens (once), or None while it is waiting or running."""
        if rid in self._done:
            return self._done.pop(rid)
        if any(r.rid == rid for r in self._live) or any(r.rid == rid for r in self._waiting):
            return None
        raise UnknownChannel(f"no request {rid}")

    def stats(self) -> dict:
        return {"waiting": len(self._waiting), "live": len(self._live), "free_pages": self.lm.free_pages, "free_slots": self.lm.free_slots,
                "reserved_pages": self._reserved}

    # ---- scheduling ------------------------------------------------------------------------------------------------
    def _admit(self) -> None:
        while self._waiting and self.lm.free_slots > 0 and self._reserved + self._waiting[0].pages <= self.lm.total_pages:
            r = self._waiting.popleft()
            r.slot = self.lm.open()
            self._reserved += r.pages
            self._live.append(r)

    def _finish(self, r: _Request, keep: bool = True) -> None:
        self.lm.close(r.slot)
        self._live.remove(r)
        self._reserved -= r.pages
        if keep:
            self._done[r.rid] = r.out

    def step(self) -> int:
        """One batch; returns the number of requests that were part of it (0: nothing to do)."""
        self._admit()
        budget, entries, sampled = self.step_tokens, [], []
        for r in self._live:                                       # decoding requests first: one token each, drawn on the device
            if not r.prefilling and budget > 0:
                entries.append((r.slot, [-1], [0]))
                sampled.append(r)
                budget -= 1
        n_decode = len(entries)
        for r in self._live:
            if r.prefilling and budget > 0:
                n = min(budget, len(r.prompt) - r.fed)
                last = r.fed + n == len(r.prompt)
                entries.append((r.slot, r.prompt[r.fed:r.fed + n], [n - 1] if last else []))
                r.fed += n
                budget -= n
                if last:
                    sampled.append(r)
        if not entries:
            return 0
        if n_decode == 0 and not sampled:
            self.lm.step(entries)
            return len(entries)
        logits = self.lm.step(entries)
        tokens = self.lm.sample(logits, [r.slot for r in sampled], [r.temp for r in sampled], [r.top_k for r in sampled], seed=self.seed).tolist()
        for r, t in zip(sampled, tokens):
            r.out.append(t)
            if len(r.out) >= r.max_new or t in r.stop:
                self._finish(r)
        # requests beyond the budget take their turn first in the next step
        if len(self._live) > self.step_tokens:
            self._live = self._live[self.step_tokens:] + self._live[:self.step_tokens]
        return len(entries)

    def generate(self, prompts: Sequence[Sequence[int]], max_new_tokens: int, temp: float = 0.0, top_k: int = 0, stop: Iterable[int] = ()) -> List[List[int]]:
        stop = list(stop)
        ids = [self.submit(p, max_new_tokens, temp, top_k, stop) for p in prompts]
        while self.step():
            pass
        return [self.pop(i) for i in ids]
