"""Sampling of the next token from a step's logits."""
from __future__ import annotations

import dataclasses
from typing import List, Optional, Sequence as Seq

import torch


@dataclasses.dataclass
class SamplingParams:
    max_tokens: int = 16
    temperature: float = 0.0                 # 0: greedy
    top_k: int = 0                           # 0: all
    top_p: float = 1.0
    seed: Optional[int] = None
    stop_token_ids: Seq[int] = ()

    def __post_init__(self):
        if self.max_tokens < 1 or self.temperature < 0 or self.top_k < 0 or not 0 < self.top_p <= 1:
            raise ValueError("invalid sampling parameters: %r" % (self,))


def filtered_probabilities(z: torch.Tensor, p: SamplingParams) -> torch.Tensor:
    """One row of logits -> probabilities after temperature, top-k and top-p (at least one token stays)."""
    z = z.float() / p.temperature
    if p.top_k and p.top_k < z.numel():
        z = torch.where(z < torch.topk(z, p.top_k).values[-1], torch.full_like(z, -float("inf")), z)
    prob = torch.softmax(z, dim=-1)
    if p.top_p < 1.0:
        v, idx = torch.sort(prob, descending=True)
        drop = torch.cumsum(v, 0) - v >= p.top_p           # mass in front of the token already reaches top_p
        drop[0] = False
        prob = prob.index_fill(0, idx[drop], 0.0)
        prob = prob / prob.sum()
    return prob


class Sampler:
    def __init__(self, model, device):
        self.model, self.device = model, device

    def generator(self, params: SamplingParams) -> Optional[torch.Generator]:
        if params.temperature == 0 or params.seed is None:
            return None
        g = torch.Generator(device=self.device)
        g.manual_seed(params.seed)
        return g

    def __call__(self, logits: torch.Tensor, params: List[SamplingParams], generators) -> List[int]:
        """One token per row of logits."""
        ids = self.model.greedy(logits)
        picked = [None if p.temperature == 0 else torch.multinomial(filtered_probabilities(logits[i], p), 1, generator=g)
                  for i, (p, g) in enumerate(zip(params, generators))]
        out = ids.tolist()
        return [t if s is None else int(s) for t, s in zip(out, picked)]
