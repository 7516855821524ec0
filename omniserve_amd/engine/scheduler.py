"""First come, first served continuous batching: every step carries one token of each running request and, with the tokens left in
its budget, portions of prompts.  When pages run out the youngest running request is put back (its tokens are recomputed later)."""
from __future__ import annotations

import dataclasses
from collections import deque
from typing import Deque, List, Optional, Tuple

from .cache import Cache, Sequence
from .sampling import SamplingParams


@dataclasses.dataclass
class Request:
    id: object
    prompt: List[int]
    params: SamplingParams
    output: List[int] = dataclasses.field(default_factory=list)
    seq: Optional[Sequence] = None
    generator: object = None
    finish_reason: Optional[str] = None

    @property
    def tokens(self) -> List[int]:
        return self.prompt + self.output

    def pending(self) -> int:
        """Tokens known but not yet run."""
        return len(self.prompt) + len(self.output) - (self.seq.length if self.seq else 0)


class Scheduler:
    def __init__(self, cache: Cache, max_batch_tokens: int):
        self.cache, self.max_batch_tokens = cache, max_batch_tokens
        self.waiting: Deque[Request] = deque()
        self.running: List[Request] = []           # oldest first

    def add(self, r: Request) -> None:
        self.waiting.append(r)

    def has_work(self) -> bool:
        return bool(self.waiting or self.running)

    def finish(self, r: Request, reason: str) -> None:
        r.finish_reason = reason
        self.running.remove(r)
        self.cache.close(r.seq)
        r.seq = None

    def abort(self, request_id) -> bool:
        for r in list(self.running):
            if r.id == request_id:
                self.finish(r, "aborted")
                return True
        for r in list(self.waiting):
            if r.id == request_id:
                self.waiting.remove(r)
                r.finish_reason = "aborted"
                return True
        return False

    def _put_back(self, r: Request) -> None:
        self.running.remove(r)
        self.cache.close(r.seq)
        r.seq = None
        self.waiting.appendleft(r)

    def _fitting(self, seq: Sequence, want: int) -> int:
        """The most of `want` tokens the free pages hold."""
        c = self.cache
        if not c.paged:
            return want
        room = (seq.pages + c.free_pages()) * c.page_size - seq.length
        return max(0, min(want, room))

    def schedule(self) -> List[Tuple[Request, int]]:
        """-> [(request, tokens to run)]; pages are reserved."""
        plan, budget = [], self.max_batch_tokens
        # single tokens first: running requests with one pending token, oldest first
        for r in list(self.running):
            if r not in self.running or r.pending() != 1 or budget == 0:
                continue
            while self.cache.missing_pages(r.seq, 1) > self.cache.free_pages():
                victim = self.running[-1]
                plan = [(q, n) for q, n in plan if q is not victim]
                self._put_back(victim)
                if victim is r:
                    break
            if r.seq is None:
                continue
            self.cache.reserve(r.seq, 1)
            plan.append((r, 1))
            budget -= 1
        # then portions of prompts under way, then new requests
        for r in self.running:
            if r.pending() > 1 and budget > 0:
                n = self._fitting(r.seq, min(r.pending(), budget))
                if n > 0:
                    self.cache.reserve(r.seq, n)
                    plan.append((r, n))
                    budget -= n
        while self.waiting and budget > 0 and self.cache.free_slots():
            r = self.waiting[0]
            seq = self.cache.open()
            n = self._fitting(seq, min(len(r.tokens), budget))
            if n == 0:
                self.cache.close(seq)
                break
            self.waiting.popleft()
            r.seq = seq
            self.running.append(r)
            self.cache.reserve(seq, n)
            plan.append((r, n))
            budget -= n
        if not plan and self.waiting and not self.running:
            raise RuntimeError("no request can start: other sequences hold every slot or page")
        if not plan and self.running:
            # several unfinished prompts hold all pages: the youngest gives way
            if len(self.running) > 1:
                self._put_back(self.running[-1])
                return self.schedule()
            raise RuntimeError("request %r does not fit the cache (%d pages)" % (self.running[0].id, self.cache.num_pages))
        return plan
