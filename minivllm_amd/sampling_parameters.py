"""Sampling parameters (src/myvllm/sampling_parameters.py:4-11)."""
from dataclasses import dataclass


@dataclass
class SamplingParams:
    temperature: float = 1.0
    max_tokens: int = 64
    ignore_eos: bool = False
    greedy: bool = False          # the most likely token: sampling at a temperature at which nothing else is ever drawn

    def __post_init__(self):
        if self.greedy:
            self.temperature = 1e-9
        assert self.temperature > 1e-10, "greedy sampling is not permitted"
