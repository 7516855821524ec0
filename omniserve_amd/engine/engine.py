"""The engine: runs steps of a model over its cache.

Two ways in, one step function (`run`):
  * `generate` / `add_request` + `step`: the scheduler forms the batches, the sampler picks tokens;
  * `open` / `run` / `close`: the caller says which sequences advance by which tokens and gets logits (replaying a trace).

Steps of single tokens only are captured in HIP graphs, one per (padded batch size, block table width)."""
from __future__ import annotations

import dataclasses
from typing import Dict, List, Optional, Sequence as Seq

import torch

from ..persistent import GraphedStep
from .batch import BatchBuilder, DecodeSlots, Entry
from .cache import Cache, Sequence
from .sampling import Sampler, SamplingParams
from .scheduler import Request, Scheduler

MAX_GRAPH_BATCH = 64


@dataclasses.dataclass
class SequenceInput:
    seq: Sequence
    tokens: Seq[int]
    want: Seq[int] = ()


@dataclasses.dataclass
class RequestOutput:
    id: object
    prompt: List[int]
    tokens: List[int]
    finish_reason: str


class Engine:
    def __init__(self, model, max_tokens: int = 65536, max_seqs: int = 16, max_batch_tokens: int = 8192, use_graphs: bool = True):
        """max_tokens: tokens the cache pool holds; max_seqs: live sequences; max_batch_tokens: tokens of one step."""
        if max_tokens < 1 or max_seqs < 1 or max_batch_tokens < max_seqs:
            raise ValueError("the engine needs room for at least one token of every sequence")
        self.model, self.device = model, torch.device(model.device)
        self.cache = Cache(model, -(-max_tokens // model.page_size), max_seqs, self.device)
        self.builder = BatchBuilder(model, self.device)
        self.scheduler = Scheduler(self.cache, max_batch_tokens)
        self.sampler = Sampler(model, self.device)
        self.use_graphs = use_graphs and model.capturable
        self._graphs: Dict[tuple, tuple] = {}
        self._next_id = 0

    # ---- sequences driven by the caller --------------------------------------------------------------------------
    def open(self) -> Sequence:
        return self.cache.open()

    def close(self, seq: Sequence) -> None:
        self.cache.close(seq)

    def run(self, inputs: List[SequenceInput]) -> Optional[torch.Tensor]:
        """One step: every sequence advances by its tokens.  Returns the wanted logits, f32 [wanted, vocab], in the order of the
        inputs and of their `want` (None when nothing is wanted); valid until the next step."""
        entries = []
        for x in inputs:
            if not x.tokens:
                raise ValueError("an entry without tokens")
            if any(not 0 <= t < self.model.vocab for t in x.tokens):
                raise ValueError("token id outside the vocabulary of %d" % self.model.vocab)
            if any(not 0 <= w < len(x.tokens) for w in x.want):
                raise ValueError("a wanted place outside the entry's tokens")
            entries.append(Entry(x.seq, x.tokens, x.want))
        if len({id(e.seq) for e in entries}) != len(entries):
            raise ValueError("a sequence appears twice in one step")
        for e in entries:
            self.cache.reserve(e.seq, len(e.tokens))
        return self._execute(entries)

    def _execute(self, entries: List[Entry]) -> Optional[torch.Tensor]:
        if not entries:
            return None
        if self.use_graphs and len(entries) <= MAX_GRAPH_BATCH and all(len(e.tokens) == 1 for e in entries):
            logits = self._decode_graph(entries)
            wanted = [i for i, e in enumerate(entries) for _ in e.want]
            if wanted != list(range(logits.shape[0])):
                logits = logits[torch.tensor(wanted, dtype=torch.int64, device=self.device)] if wanted else None
        else:
            batch, places = self.builder.build(entries)
            logits = self.model.forward(batch, self.cache)
            order = sorted(range(len(places)), key=lambda k: places[k][0])        # stable: `want` order inside an entry
            if order != list(range(len(places))):
                logits = logits[torch.tensor(order, dtype=torch.int64, device=self.device)]
        for e in entries:
            self.cache.advance(e.seq, len(e.tokens))
        return logits

    def _decode_graph(self, entries: List[Entry]) -> torch.Tensor:
        places, width = 1, 4
        while places < len(entries):
            places *= 2
        while width < max(e.seq.pages for e in entries):
            width *= 2
        key = (places, width)
        if key not in self._graphs:
            slots, out = DecodeSlots(self.builder, places, width), {}

            def step():
                out["logits"] = self.model.forward(slots.batch, self.cache)

            graph = GraphedStep(step, self.device)
            graph.capture()                         # every place is empty: neither the cache nor the state is touched
            self._graphs[key] = (slots, graph, out)
        slots, graph, out = self._graphs[key]
        slots.fill(entries)
        graph.run()
        return out["logits"][:len(entries)]

    # ---- requests ------------------------------------------------------------------------------------------------
    def add_request(self, prompt: Seq[int], params: Optional[SamplingParams] = None, request_id=None):
        prompt, params = [int(t) for t in prompt], params or SamplingParams()
        if not prompt:
            raise ValueError("an empty prompt")
        if any(not 0 <= t < self.model.vocab for t in prompt):
            raise ValueError("token id outside the vocabulary of %d" % self.model.vocab)
        if request_id is None:
            request_id, self._next_id = self._next_id, self._next_id + 1
        self.scheduler.add(Request(request_id, prompt, params, generator=self.sampler.generator(params)))
        return request_id

    def abort(self, request_id) -> bool:
        return self.scheduler.abort(request_id)

    def has_work(self) -> bool:
        return self.scheduler.has_work()

    def step(self) -> List[RequestOutput]:
        """One engine step; returns the requests that finished in it."""
        plan = self.scheduler.schedule()
        if not plan:
            return []
        entries, sampled = [], []
        for r, n in plan:
            at = r.seq.length
            done = n == r.pending()                # the last known token runs: its logits give the next one
            entries.append(Entry(r.seq, r.tokens[at:at + n], [n - 1] if done else []))
            if done:
                sampled.append(r)
        logits = self._execute(entries)
        finished = []
        if sampled:
            for r, t in zip(sampled, self.sampler(logits, [r.params for r in sampled], [r.generator for r in sampled])):
                r.output.append(t)
                if t in r.params.stop_token_ids:
                    self.scheduler.finish(r, "stop")
                elif len(r.output) >= r.params.max_tokens:
                    self.scheduler.finish(r, "length")
                if r.finish_reason:
                    finished.append(RequestOutput(r.id, r.prompt, r.output, r.finish_reason))
        return finished

    def generate(self, prompts: Seq[Seq[int]], params=None) -> List[RequestOutput]:
        """Runs the prompts to their end; outputs in the order of the prompts.  params: one for all, or one per prompt."""
        each = list(params) if isinstance(params, (list, tuple)) else [params] * len(prompts)
        ids = [self.add_request(p, q) for p, q in zip(prompts, each)]
        done = {}
        while self.has_work():
            for o in self.step():
                done[o.id] = o
        return [done[i] for i in ids]
