"""Counterparts of the reference's small layers around the attention path, as chains of PyTorch-ROCm tensor
operations and, with ``fused=True``, as single HIP launches (minivllm_amd.layers.fused): RMSNorm with fused residual (layers/layernorm.py:9-28), NeoX half-split RoPE
(layers/rotary_embedding.py:4-83), SiluAndMul (layers/activation.py:15-18) and the temperature /
exponential-race sampler (layers/sampler.py:14-19)."""
from __future__ import annotations

import math

import torch
import torch.nn as nn
import torch.nn.functional as F

from minivllm_amd.layers.fused import add_rms_norm, gelu_tanh, linear_small_m, linear_small_m_takes, silu_and_mul


class Linear(nn.Linear):
    """``nn.Linear`` (layers/linear.py) whose calls with at most ``small_rows`` rows (a decode step) run as one HIP
    launch built for that size (``linear_small_m``); everything else, prefill included, is the library GEMM."""

    def __init__(self, in_features: int, out_features: int, bias: bool = True, small_rows: int = 0):
        super().__init__(in_features, out_features, bias=bias)
        self.small_rows = small_rows

    def forward(self, x, gelu: bool = False):
        """``gelu``: the result through the tanh form of gelu."""
        if self.small_rows and linear_small_m_takes(x, self.weight, self.small_rows):
            return linear_small_m(x, self.weight, self.bias, gelu)
        y = F.linear(x, self.weight, self.bias)
        return gelu_tanh(y, out=y) if gelu else y


class RMSNorm(nn.Module):
    """x / sqrt(mean(x^2) + eps) * weight over the last dim, optionally after adding a residual
    (layers/layernorm.py:9-28).  ``fused=True`` runs it as one HIP launch (``add_rms_norm``), otherwise as the
    chain of tensor operations; both round where the chain rounds."""

    def __init__(self, size: int, eps: float = 1e-6, fused: bool = False):
        super().__init__()
        self.weight = nn.Parameter(torch.ones(size))
        self.eps = eps
        self.fused = fused
        self._w32 = None

    def weight_fp32(self):
        """float32 copy of the weight for the HIP kernels (made once; weights do not change while serving)."""
        if self._w32 is None or self._w32.device != self.weight.device:
            self._w32 = self.weight.detach().float().contiguous()
        return self._w32

    def _norm(self, x):
        xf = x.float()
        xf = xf / torch.sqrt(xf.pow(2).mean(dim=-1, keepdim=True) + self.eps)
        return (xf * self.weight.float()).to(x.dtype)

    def forward(self, x, residual=None):
        if self.fused and x.dim() == 2:
            return add_rms_norm(x, self.weight_fp32(), self.eps, residual)
        if residual is None:
            return self._norm(x)
        x = x + residual
        return self._norm(x), x


class RotaryEmbedding(nn.Module):
    def __init__(self, base: float, rotary_dim: int, max_position: int):
        super().__init__()
        self.base, self.rotary_dim, self.max_position = base, rotary_dim, max_position
        self.register_buffer("cos_sin_cache", self._table(), persistent=False)

    def _table(self):
        inv_freq = 1.0 / (self.base ** (torch.arange(0, self.rotary_dim, 2, dtype=torch.float32) / self.rotary_dim))
        freqs = torch.outer(torch.arange(self.max_position, dtype=torch.float32), inv_freq)
        return torch.cat([freqs.cos(), freqs.sin()], dim=-1)

    def _apply(self, fn, recurse=True):
        # the table stays float32 whatever dtype the model is cast to (rotary_embedding.py:61-70 builds it
        # from float positions): rebuild it on the device the cast left it on
        super()._apply(fn, recurse)
        self.cos_sin_cache = self._table().to(self.cos_sin_cache.device)
        return self

    @staticmethod
    def _rotate(x, cos, sin):
        x1, x2 = x.float().chunk(2, dim=-1)
        return torch.cat([x1 * cos - x2 * sin, x1 * sin + x2 * cos], dim=-1).to(x.dtype)

    def forward(self, positions, query, key):
        cos, sin = self.cos_sin_cache[positions].chunk(2, dim=-1)      # (T, D/2) each, fp32
        cos, sin = cos.unsqueeze(1), sin.unsqueeze(1)
        return self._rotate(query, cos, sin), self._rotate(key, cos, sin)


def rotary_pair_table(base: float, dims: int, max_position: int, scaling: dict | None = None) -> torch.Tensor:
    """float32 (max_position, dims / 2, 2): cos and sin of position * base^(-2 i / dims), angles in double precision.

    ``scaling`` (``factor``, ``low``, ``high``, ``original``) stretches the slow pairs: wavelengths beyond original / low
    by ``factor``, those below original / high not at all, a blend linear in original / wavelength between them.  With
    ``fast`` and ``slow`` instead (YaRN) the blend is linear in the pair's number, between the pairs that turn ``fast`` and
    ``slow`` times over the original context, and cos and sin are multiplied by 0.1 ln(factor) + 1."""
    freq = float(base) ** (-torch.arange(0, dims, 2, dtype=torch.float64) / dims)
    amplitude = 1.0
    if scaling is not None and "fast" in scaling:
        def pair_of(turns):
            return dims * math.log(scaling["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

        lo, hi = max(math.floor(pair_of(scaling["fast"])), 0), min(math.ceil(pair_of(scaling["slow"])), dims - 1)
        stretch = ((torch.arange(dims // 2, dtype=torch.float64) - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
        freq = freq / scaling["factor"] * stretch + freq * (1.0 - stretch)
        amplitude = 0.1 * math.log(scaling["factor"]) + 1.0
    elif scaling is not None:
        turns = scaling["original"] * freq / (2 * math.pi)                 # of a pair over the original context
        keep = ((turns - scaling["low"]) / (scaling["high"] - scaling["low"])).clamp(0.0, 1.0) if (
            scaling["high"] != scaling["low"]) else (turns > scaling["high"]).double()
        freq = (1.0 - keep) * freq / scaling["factor"] + keep * freq
    angle = torch.outer(torch.arange(max_position, dtype=torch.float64), freq)
    return (torch.stack([angle.cos(), angle.sin()], dim=-1) * amplitude).float().contiguous()


class SiluAndMul(nn.Module):
    def __init__(self, fused: bool = False):
        super().__init__()
        self.fused = fused

    def forward(self, x):
        if self.fused and x.dim() == 2:
            return silu_and_mul(x)
        a, b = x.chunk(2, dim=-1)
        return F.silu(a) * b


class Sampler(nn.Module):
    """argmax(softmax(logits / T) / E), E ~ Exp(1): one draw from the tempered distribution."""

    def forward(self, logits, temperatures, generator=None):
        probs = torch.softmax(logits.float() / temperatures.unsqueeze(-1), dim=-1)
        noise = torch.empty_like(probs).exponential_(1.0, generator=generator).clamp_min_(1e-10)
        return probs.div_(noise).argmax(dim=-1)
