"""Token sampling from a step's logits."""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import List, Optional

import torch


@dataclass
class SamplingParams:
    max_tokens: int = 16
    temperature: float = 0.0     # 0 = greedy
    top_k: int = 0               # 0 = all
    top_p: float = 1.0
    seed: Optional[int] = None
    stop_ids: List[int] = field(default_factory=list)

    def __post_init__(self):
        if self.max_tokens < 1 or self.temperature < 0 or self.top_k < 0 or not 0 < self.top_p <= 1:
            raise ValueError(f"invalid sampling parameters: {self}")


class Sampler:
    """One per request: holds the request's generator."""

    def __init__(self, params: SamplingParams, device):
        self.params = params
        self._gen = None
        if params.temperature > 0:
            self._gen = torch.Generator(device=device)
            if params.seed is not None:
                self._gen.manual_seed(params.seed)
            else:
                self._gen.seed()

    def sample(self, logits: torch.Tensor) -> int:
        """logits [vocab] -> token id."""
        p = self.params
        if p.temperature == 0:
            return int(torch.argmax(logits))
        x = logits.float() / p.temperature
        order = torch.argsort(x, descending=True, stable=True)
        probs = torch.softmax(x[order], dim=-1)
        keep = probs.numel()
        if p.top_k:
            keep = min(keep, p.top_k)
        if p.top_p < 1:   # the smallest prefix that reaches top_p
            keep = min(keep, int((probs.cumsum(0) < p.top_p).sum()) + 1)
        pick = torch.multinomial(probs[:keep], 1, generator=self._gen)
        return int(order[pick])
