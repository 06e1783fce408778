"""Operators of recurrent layers: gate projections in fp32, the mLSTM's matrix-memory recurrence and the one with a constant
decay per head.

``MlstmState`` holds the state of every slot of one layer; ``mlstm`` runs a ragged step through it and applies the
per-head norm and output gate.  ``DecayMemoryState`` and ``decay_memory`` are the same for constant decays, ``gated_row_norm``
is what follows there.  All of it calls libminivllm_amd.so on the current torch stream."""
from __future__ import annotations

import math
from dataclasses import dataclass

import torch

from minivllm_amd import _C

__all__ = ["DecayMemoryState", "MlstmState", "decay_memory", "gate_linear", "gated_row_norm", "mlstm"]

DEN_FLOOR = 1e-6          # added to the normaliser max(|n . q|, exp(-m))


def _ptr(t):
    return 0 if t is None else t.data_ptr()


@dataclass
class MlstmState:
    s: torch.Tensor       # (slots, H, dim, vdim) float32
    n: torch.Tensor       # (slots, H, dim)
    m: torch.Tensor       # (slots, H)

    @classmethod
    def allocate(cls, slots: int, heads: int, dim: int, vdim: int, device) -> "MlstmState":
        new = lambda *shape: torch.zeros(slots, heads, *shape, dtype=torch.float32, device=device)
        return cls(new(dim, vdim), new(dim), new())


def gate_linear(x: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor | None, split: int, cap: float) -> torch.Tensor:
    """float32 (T, N) = act(x weight^T + bias): columns below ``split`` through cap * tanh(z / cap), the others through
    logsigmoid of that.  x (T, K) and weight (N, K) in one dtype (bf16 / fp32), bias float32 (N,)."""
    _C.require_cuda(x, weight, bias)
    rows, k = x.shape
    n = weight.shape[0]
    if weight.dtype != x.dtype or weight.shape[1] != k or not weight.is_contiguous() or (k > 1 and x.stride(1) != 1):
        raise ValueError("x (T, K) with dense rows and a contiguous weight (N, K) of one dtype expected")
    if bias is not None and (bias.dtype != torch.float32 or bias.numel() != n or not bias.is_contiguous()):
        raise ValueError(f"bias must be contiguous float32 ({n},)")
    out = torch.empty((rows, n), dtype=torch.float32, device=x.device)
    st = _C.load().mvllm_gate_linear(_ptr(out), _ptr(x), x.stride(0) if rows > 1 else k, _ptr(weight), _ptr(bias), rows, n, k,
                                     split, float(cap), _C.dtype_code(x.dtype), _C.current_stream_ptr(x.device))
    _C.check(st, "gate_linear")
    return out


def chunked_takes(proj: torch.Tensor, dim: int, vdim: int) -> bool:
    """Whether the block form is built for this layer (otherwise every row goes through the recurrence in turn)."""
    return (proj.dtype == torch.bfloat16 and dim % 8 == 0 and vdim % 8 == 0 and dim <= 256 and proj.data_ptr() % 16 == 0
            and proj.shape[1] % 8 == 0 and (proj.shape[0] == 1 or proj.stride(0) % 8 == 0))


def mlstm(step, proj: torch.Tensor, gates: torch.Tensor, gate_col: int, weight: torch.Tensor, state: MlstmState,
          eps: float) -> torch.Tensor:
    """The mLSTM mixer between its projections: (T, H * vdim) = rms(recurrence) * weight * sigmoid(gate).

    proj (T, *): q (H, dim) | k (H, dim) | v (H, vdim) at its start and the output gate's H * vdim columns at ``gate_col``;
    gates float32 (T, 2 H): log input and log forget gates; weight float32 (H * vdim,)."""
    _C.require_cuda(proj, gates, weight, state.s)
    slots, heads, dim, vdim = state.s.shape
    rows = proj.shape[0]
    if proj.dim() != 2 or proj.stride(1) != 1 or gate_col < heads * (2 * dim + vdim) or proj.shape[1] < gate_col + heads * vdim:
        raise ValueError("proj must hold q, k, v and, from gate_col on, the output gate")
    if gates.dtype != torch.float32 or tuple(gates.shape) != (rows, 2 * heads) or not gates.is_contiguous():
        raise ValueError(f"gates must be contiguous float32 ({rows}, {2 * heads})")
    if weight.dtype != torch.float32 or weight.numel() != heads * vdim or not weight.is_contiguous():
        raise ValueError(f"weight must be contiguous float32 ({heads * vdim},)")
    if step.num_tokens != rows:
        raise ValueError("the step's rows and proj's differ")
    dev, code = proj.device, _C.dtype_code(proj.dtype)
    stream = _C.current_stream_ptr(dev)
    stride = proj.stride(0) if rows > 1 else proj.shape[1]
    num = torch.empty((rows, heads, vdim), dtype=torch.float32, device=dev)
    den = torch.empty((rows, heads), dtype=torch.float32, device=dev)
    m_next = torch.empty((step.num_entries, heads), dtype=torch.float32, device=dev)
    out = torch.empty((rows, heads * vdim), dtype=proj.dtype, device=dev)
    lib = _C.load()
    scale = dim ** -0.5
    common = (_ptr(num), _ptr(den), _ptr(m_next), _ptr(proj), stride, _ptr(gates), _ptr(state.s), _ptr(state.n), _ptr(state.m),
              _ptr(step.cu_seqlens), _ptr(step.state_slots), _ptr(step.positions))
    blocks = step.segments is not None and chunked_takes(proj, dim, vdim)
    row_by_row = step.num_short if blocks else step.num_entries
    if row_by_row:
        _C.check(lib.mvllm_mlstm_recurrent(*common, row_by_row, heads, dim, vdim, scale, DEN_FLOOR, code, stream),
                 "mlstm_recurrent")
    if blocks:
        count = step.segments.shape[0]
        nbytes = lib.mvllm_mlstm_chunked_workspace_bytes(count, heads, dim, vdim) if step.split else 0
        ws = torch.empty(nbytes, dtype=torch.uint8, device=dev) if nbytes else None
        _C.check(lib.mvllm_mlstm_chunked(*common, _ptr(step.segments), count, int(step.split), heads, dim, vdim, scale,
                                         DEN_FLOOR, code, _ptr(ws), nbytes, stream), "mlstm_chunked")
    _C.check(lib.mvllm_mlstm_output(
        _ptr(out), _ptr(num), _ptr(den), _ptr(weight), proj.data_ptr() + gate_col * proj.element_size(), stride, float(eps),
        _ptr(m_next), _ptr(state.m), _ptr(step.cu_seqlens), _ptr(step.row_entry), _ptr(step.state_slots), rows, heads, vdim,
        code, stream), "mlstm_output")
    return out


@dataclass
class DecayMemoryState:
    s: torch.Tensor            # (slots, H, dim, vdim) float32
    decay: torch.Tensor        # (H,) float32
    log_decay: torch.Tensor    # its logarithm, taken in double precision

    @classmethod
    def allocate(cls, slots: int, decay: list, dim: int, vdim: int, device) -> "DecayMemoryState":
        if any(not 0.0 <= d <= 1.0 for d in decay):
            raise ValueError("decays must lie between 0 and 1")
        f32 = lambda x: torch.tensor(x, dtype=torch.float32, device=device)
        logs = [math.log(d) if d > 1e-300 else -1e4 for d in decay]          # exp(-1e4) is zero, and 0 * -1e4 is too
        return cls(torch.zeros(slots, len(decay), dim, vdim, dtype=torch.float32, device=device), f32(decay), f32(logs))


def decay_memory(step, proj: torch.Tensor, state: DecayMemoryState, silu: bool = True) -> torch.Tensor:
    """float32 (T, H * vdim): o = S^T q with S <- decay S + k v^T along every entry of the step, from the slots' states.

    proj (T, *): q (H, dim) | k (H, dim) | v (H, vdim) at its start; ``silu``: each of them through z * sigmoid(z) first."""
    _C.require_cuda(proj, state.s)
    slots, heads, dim, vdim = state.s.shape
    rows = proj.shape[0]
    if proj.dim() != 2 or proj.stride(1) != 1 or proj.shape[1] < heads * (2 * dim + vdim):
        raise ValueError("proj must hold q, k and v")
    if step.num_tokens != rows:
        raise ValueError("the step's rows and proj's differ")
    dev, code = proj.device, _C.dtype_code(proj.dtype)
    stream = _C.current_stream_ptr(dev)
    stride = proj.stride(0) if rows > 1 else proj.shape[1]
    num = torch.empty((rows, heads * vdim), dtype=torch.float32, device=dev)
    lib = _C.load()
    blocks = step.segments is not None and chunked_takes(proj, dim, vdim)
    row_by_row = step.num_short if blocks else step.num_entries
    if row_by_row:
        _C.check(lib.mvllm_decay_memory_recurrent(
            _ptr(num), _ptr(proj), stride, _ptr(state.decay), _ptr(state.s), _ptr(step.cu_seqlens), _ptr(step.state_slots),
            _ptr(step.positions), row_by_row, heads, dim, vdim, int(silu), code, stream), "decay_memory_recurrent")
    if blocks:
        count = step.segments.shape[0]
        nbytes = lib.mvllm_decay_memory_chunked_workspace_bytes(count, heads, dim, vdim) if step.split else 0
        ws = torch.empty(nbytes, dtype=torch.uint8, device=dev) if nbytes else None
        _C.check(lib.mvllm_decay_memory_chunked(
            _ptr(num), _ptr(proj), stride, _ptr(state.log_decay), _ptr(state.s), _ptr(step.cu_seqlens), _ptr(step.state_slots),
            _ptr(step.positions), _ptr(step.segments), count, int(step.split), heads, dim, vdim, int(silu), code, _ptr(ws),
            nbytes, stream), "decay_memory_chunked")
    return num


def gated_row_norm(x: torch.Tensor, weight: torch.Tensor, gate: torch.Tensor, eps: float) -> torch.Tensor:
    """rms(x) * weight * sigmoid(gate) over whole rows: x float32 (T, W) contiguous, weight float32 (W,), gate (T, W) with
    dense rows in the result's dtype."""
    _C.require_cuda(x, weight, gate)
    rows, width = x.shape
    if x.dtype != torch.float32 or not x.is_contiguous() or weight.dtype != torch.float32 or weight.numel() != width \
            or not weight.is_contiguous() or tuple(gate.shape) != (rows, width) or gate.stride(1) != 1:
        raise ValueError("x (T, W) and weight (W,) contiguous float32, gate (T, W) with dense rows expected")
    out = torch.empty((rows, width), dtype=gate.dtype, device=x.device)
    st = _C.load().mvllm_gated_row_norm(_ptr(out), width, _ptr(x), _ptr(weight), _ptr(gate), gate.stride(0) if rows > 1 else width,
                                        float(eps), rows, width, _C.dtype_code(gate.dtype), _C.current_stream_ptr(x.device))
    _C.check(st, "gated_row_norm")
    return out
