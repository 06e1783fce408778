"""Mixture of experts: router, plan and products as operators over libminivllm_amd.so, and the feed-forward module.

The module returns the experts' results unsummed (``ExpertOutput``): whoever adds the feed-forward to the residual reads
them with their weights (``layers.fused.stream_norm``)."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch
import torch.nn as nn

from minivllm_amd import _C
from minivllm_amd.layers.recurrent import gate_linear
from minivllm_amd.models.qwen3 import Qwen3MLP
from minivllm_amd.utils.padding import pad_to, round_up

__all__ = ["ExpertOutput", "ExpertPlan", "SparseExperts", "moe_route", "moe_route_softmax", "moe_plan", "moe_linear", "interleave_gate_up"]

FEW_PAIRS = 16             # (token, choice) pairs up to which the products run without a plan


def _ptr(t):
    return 0 if t is None else t.data_ptr()


@dataclass
class ExpertOutput:
    """y[t] = sum_k weights[t, k] parts[part_row[t, k]] + sigmoid(gate[t]) shared[t]; a choice whose id is negative counts with
    inputs[t]."""
    parts: torch.Tensor                       # (pairs, >= width)
    weights: torch.Tensor                     # float32 (T, top)
    part_row: Optional[torch.Tensor] = None   # int32 (T * top,), None: pair t * top + k
    shared: Optional[torch.Tensor] = None     # (T, width)
    gate: Optional[torch.Tensor] = None       # float32 (T,), any stride; None: 1
    ids: Optional[torch.Tensor] = None        # int32 (T, top), None: every choice is an expert
    inputs: Optional[torch.Tensor] = None     # (T, >= width)


class ExpertPlan:
    """Pairs sorted by expert (device memory only; the host never learns how many rows an expert has)."""

    def __init__(self, ids: torch.Tensor, experts: int):
        self.pairs = ids.numel()
        nbytes = int(_C.load().mvllm_moe_plan_bytes(self.pairs, experts))
        self.data = torch.empty(nbytes // 4, dtype=torch.int32, device=ids.device)
        st = _C.load().mvllm_moe_plan(_ptr(self.data), nbytes, _ptr(ids), self.pairs, experts, _C.current_stream_ptr(ids.device))
        _C.check(st, "moe_plan")

    @property
    def place(self) -> torch.Tensor:
        """Sorted place of every pair."""
        return self.data[:self.pairs]


def moe_route(logits: torch.Tensor, correction: torch.Tensor | None, experts: int, top: int, groups: int = 1, keep: int = 1):
    """(ids int32 (T, top), weights float32 (T, top)) from float32 logits (T, >= experts)."""
    _C.require_cuda(logits, correction)
    if logits.dtype != torch.float32 or logits.stride(1) != 1 or logits.shape[1] < experts:
        raise ValueError("logits must be float32 with dense rows, one column per expert")
    if correction is not None and (correction.dtype != torch.float32 or correction.numel() != experts or not correction.is_contiguous()):
        raise ValueError(f"correction must be contiguous float32 ({experts},)")
    t = logits.shape[0]
    ids = torch.empty((t, top), dtype=torch.int32, device=logits.device)
    weights = torch.empty((t, top), dtype=torch.float32, device=logits.device)
    st = _C.load().mvllm_moe_route(_ptr(ids), _ptr(weights), _ptr(logits), logits.stride(0) if t > 1 else logits.shape[1],
                                   _ptr(correction), t, experts, top, groups, keep, _C.current_stream_ptr(logits.device))
    _C.check(st, "moe_route")
    return ids, weights


def moe_route_softmax(logits: torch.Tensor, correction: torch.Tensor | None, experts: int, identity: int, top: int,
                      renormalize: bool = False):
    """(ids int32 (T, top), weights float32 (T, top)): the largest softmax(logits) + correction, weighted by the softmax.  The last
    ``identity`` of the experts + identity columns stand for no expert; their id is -1."""
    _C.require_cuda(logits, correction)
    n = experts + identity
    if logits.dtype != torch.float32 or logits.stride(1) != 1 or logits.shape[1] < n:
        raise ValueError("logits must be float32 with dense rows, one column per expert and identity expert")
    if correction is not None and (correction.dtype != torch.float32 or correction.numel() != n or not correction.is_contiguous()):
        raise ValueError(f"correction must be contiguous float32 ({n},)")
    t = logits.shape[0]
    ids = torch.empty((t, top), dtype=torch.int32, device=logits.device)
    weights = torch.empty((t, top), dtype=torch.float32, device=logits.device)
    st = _C.load().mvllm_moe_route_softmax(_ptr(ids), _ptr(weights), _ptr(logits), logits.stride(0) if t > 1 else logits.shape[1],
                                           _ptr(correction), t, experts, identity, top, int(renormalize), _C.current_stream_ptr(logits.device))
    _C.check(st, "moe_route_softmax")
    return ids, weights


def moe_plan(ids: torch.Tensor, experts: int) -> ExpertPlan:
    _C.require_cuda(ids)
    if ids.dtype != torch.int32 or not ids.is_contiguous():
        raise ValueError("ids must be contiguous int32")
    return ExpertPlan(ids, experts)


def moe_linear(x: torch.Tensor, weight: torch.Tensor, ids: torch.Tensor, plan: ExpertPlan | None = None, per_token: int = 0,
               glu: bool | tuple = False) -> torch.Tensor:
    """Row p = x[row of p] W_e^T for every (token, choice) pair of ``ids`` (T, top), e its expert; with ``glu`` silu(gate) * up, with
    ``glu`` = (alpha, limit, shift) the clamped form of ``layers.fused.gated_unit``.  Pairs with negative ids have no row.

    With a plan rows are in its sorted order, without in the pairs'.  ``per_token`` > 0: pair p reads row p / per_token of x,
    0: row p of x is row p's own (an earlier product's).  weight (E, N, K), with ``glu`` as ``interleave_gate_up`` makes it."""
    _C.require_cuda(x, weight, ids)
    experts, n, k = weight.shape
    pairs = ids.numel()
    if x.dim() != 2 or x.shape[1] != k or x.stride(1) != 1 or weight.dtype != x.dtype or not weight.is_contiguous():
        raise ValueError(f"x (*, {k}) with dense rows and a contiguous weight of its dtype expected")
    if ids.dtype != torch.int32 or not ids.is_contiguous() or x.shape[0] * max(per_token, 1) != pairs:
        raise ValueError("ids must be contiguous int32 and x have a row for every token or pair")
    if plan is not None and plan.pairs != pairs:
        raise ValueError("the plan is of other ids")
    out = torch.empty((pairs, n // 2 if glu else n), dtype=x.dtype, device=x.device)
    head = (_ptr(out), out.shape[1], _ptr(x), x.stride(0) if x.shape[0] > 1 else k, _ptr(weight), _ptr(ids),
            _ptr(plan.data if plan is not None else None), pairs, experts, n, k, per_token)
    tail = (_C.dtype_code(x.dtype), _C.current_stream_ptr(x.device))
    if isinstance(glu, tuple):
        st = _C.load().mvllm_moe_linear_clamped(*head, *(float(c) for c in glu), *tail)
    else:
        st = _C.load().mvllm_moe_linear(*head, int(glu), *tail)
    _C.check(st, "moe_linear")
    return out


def interleave_gate_up(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
    """(F, K) gate and up rows in turns of 32, F a multiple of 32."""
    f, k = gate.shape
    return torch.stack([gate.view(f // 32, 32, k), up.view(f // 32, 32, k)], dim=1).reshape(2 * f, k)


class SparseExperts(nn.Module):
    """``experts`` feed-forwards silu(gate) * up of size ``ff``, ``top`` of them per token, and optionally a shared one behind
    a gate of one number per token.  Inputs are ``inputs`` wide (zeros past the model's width).

    ``softmax``: scores are a softmax over experts and ``identity`` further ones that hand their input on, and weights stay as
    they are; otherwise sigmoids, weights normalized.  ``glu``: (alpha, limit, shift) of clamped gated units."""

    ALIGN = 64             # the products' step along K

    def __init__(self, width: int, inputs: int, experts: int, top: int, ff: int, groups: int = 1, keep: int = 1,
                 shared_ff: int = 0, shared_gate: bool = True, small_rows: int = 0, softmax: bool = False, identity: int = 0,
                 glu: tuple | None = None):
        super().__init__()
        if identity and not softmax:
            raise ValueError("identity experts take a softmax router")
        self.softmax, self.identity, self.glu = softmax, identity, glu if glu is not None else True
        self.width, self.inputs, self.experts, self.top, self.groups, self.keep = width, inputs, experts, top, groups, keep
        self.ff = round_up(ff, self.ALIGN)
        self.shared_gate = shared_gate and shared_ff > 0
        self.shared_ff = round_up(shared_ff, 16) if shared_ff else 0
        if shared_ff:
            with torch.device("meta"):
                self.shared = Qwen3MLP(inputs, self.shared_ff, False, True, small_rows)
        else:
            self.shared = None
        self.correction = None

    @torch.no_grad()
    def load(self, get, matrix):
        """``get(name)``: checkpoint tensor, ``matrix(t)``: a product's weight on the device in the model's type."""
        def expert(e):
            gate, up = (pad_to(matrix(get(f"e{e}.{n}")), self.ff, self.inputs) for n in ("gate", "up"))
            return interleave_gate_up(gate, up), pad_to(matrix(get(f"e{e}.down")), round_up(self.width, 16), self.ff)

        first = expert(0)
        self.gate_up = first[0].new_empty((self.experts, *first[0].shape))
        self.down = first[1].new_empty((self.experts, *first[1].shape))
        for e in range(self.experts):
            self.gate_up[e], self.down[e] = first if e == 0 else expert(e)
        rows = [get("router")] + ([get("shared.sg")] if self.shared_gate else [])
        self.router = pad_to(torch.cat([matrix(r) for r in rows]), None, self.inputs)
        self.correction = get("correction").to(device=self.router.device, dtype=torch.float32).contiguous()
        if self.shared is not None:
            gate, up = (pad_to(matrix(get(f"shared.{n}")), self.shared_ff, self.inputs) for n in ("gate", "up"))
            self.shared.gate_up.weight = nn.Parameter(torch.cat([gate, up]), requires_grad=False)
            self.shared.gate_down.weight = nn.Parameter(pad_to(matrix(get("shared.down")), None, self.shared_ff), requires_grad=False)

    def forward(self, h) -> ExpertOutput:
        logits = gate_linear(h, self.router, None, self.router.shape[0], 0.0)
        if self.softmax:
            ids, weights = moe_route_softmax(logits, self.correction, self.experts, self.identity, self.top)
        else:
            ids, weights = moe_route(logits, self.correction, self.experts, self.top, self.groups, self.keep)
        pairs = ids.numel()
        plan = None
        if h.dtype != torch.bfloat16 or pairs > FEW_PAIRS:
            plan = moe_plan(ids, self.experts)
        act = moe_linear(h, self.gate_up, ids, plan, self.top, glu=self.glu)
        parts = moe_linear(act, self.down, ids, plan)
        out = ExpertOutput(parts, weights, None if plan is None else plan.place)
        if self.identity:
            out.ids, out.inputs = ids, h
        if self.shared is not None:
            out.shared = self.shared(h)
            out.gate = logits[:, self.experts] if self.shared_gate else None
        return out
