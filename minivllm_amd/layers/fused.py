"""Fused caller-side operator in front of the attention kernels.

``qk_norm_rope_store`` does in one HIP launch what the reference's ``Qwen3Attention.forward`` does with
three modules per layer and step (src/myvllm/models/qwen3.py:104-110): the shared-gamma RMSNorm of q and k
(layers/layernorm.py:9-17), the half-split rotary embedding (layers/rotary_embedding.py:4-23, 77-83) and
``store_kvcache`` of the rotated k and of v (layers/attention.py:67-108).  It reads q, k and v as the three
column slices of the packed QKV projection output (no copies) and calls libminivllm_amd.so on the current
torch stream; there is no PyTorch fallback.

``sample_tokens`` is the reference's ``SamplerLayer.forward`` (layers/sampler.py:14-19) as one launch over the
LM-head output, with the Exp(1) noise drawn inside the kernel (Philox4x32-10) or passed in.
"""
from __future__ import annotations

import math

import torch

from minivllm_amd import _C

__all__ = ["qk_norm_rope_store", "sample_tokens", "sample_tokens_into", "decode_advance", "add_rms_norm", "silu_and_mul", "linear_small_m", "linear_small_m_takes", "norm_linear_small_m", "norm_linear_small_m_takes",
           "lm_head_sample", "lm_head_sample_takes", "lm_head_sample_workspace_bytes", "norm_conv", "head_rope_store",
           "head_unrotate_gate", "chunk_decode_step", "stream_embed_norm", "stream_norm", "gated_unit", "gelu_tanh", "post_norm",
           "embed_rows"]


def _ptr(t):
    return 0 if t is None else t.data_ptr()


def _rows(name, t, heads, head_dim):
    """(T, heads, head_dim) view whose (head, dim) part is dense; returns the token stride in elements."""
    if t.dim() != 3 or tuple(t.shape[1:]) != (heads, head_dim):
        raise ValueError(f"{name} must be (num_tokens, {heads}, {head_dim}), got {tuple(t.shape)}")
    if t.shape[0] > 1 and (t.stride(2) != 1 or t.stride(1) != head_dim):
        raise ValueError(f"{name}: heads and head_dim must be contiguous inside a token row")
    return t.stride(0) if t.shape[0] > 1 else heads * head_dim


def qk_norm_rope_store(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, positions: torch.Tensor,
                       cos_sin_cache: torch.Tensor, gamma: torch.Tensor | None = None, eps: float = 1e-6,
                       slot_mapping: torch.Tensor | None = None, k_cache: torch.Tensor | None = None,
                       v_cache: torch.Tensor | None = None, k_scale: torch.Tensor | None = None,
                       v_scale: torch.Tensor | None = None, need_kv: bool = True):
    """RMSNorm(q), RMSNorm(k) with one gamma over head_dim (skipped when ``gamma`` is None), rotary embedding
    of both at ``positions``, and the cache store of the rotated k and of v at ``slot_mapping``.

    q: (T, Hq, D); k, v: (T, Hkv, D), token rows may be strided (slices of the QKV projection);
    positions int64 (T,); cos_sin_cache float32 (max_position, D) = cos | sin; gamma float32 (D,);
    caches (num_blocks, block_size, Hkv, D) in q's dtype, or int8 with float32 k_scale / v_scale
    (num_blocks, block_size, Hkv).  ``slot_mapping`` None stores nothing.
    Returns (q_out, k_out, v_out) contiguous; k_out and v_out are None unless ``need_kv`` (prefill reads
    them, decode reads the cache).
    """
    _C.require_cuda(q, k, v, positions, cos_sin_cache)
    if q.dim() != 3 or k.dim() != 3:
        raise ValueError("q, k and v must be (num_tokens, heads, head_dim)")
    num_tokens, num_heads, head_dim = q.shape
    num_kv_heads = k.shape[1]
    if k.dtype != q.dtype or v.dtype != q.dtype:
        raise ValueError("q, k and v must share one dtype")
    if k.shape[0] != num_tokens or v.shape != k.shape:
        raise ValueError("q, k and v must have the same number of tokens and k, v the same shape")
    q_stride = _rows("q", q, num_heads, head_dim)
    k_stride = _rows("k", k, num_kv_heads, head_dim)
    v_stride = _rows("v", v, num_kv_heads, head_dim)
    if positions.numel() != num_tokens:
        raise ValueError("positions must have one entry per token")
    if positions.dtype != torch.int64:
        positions = positions.to(torch.int64)
    positions = positions.contiguous()
    if cos_sin_cache.dtype != torch.float32 or cos_sin_cache.dim() != 2 or cos_sin_cache.shape[1] != head_dim \
            or not cos_sin_cache.is_contiguous():
        raise ValueError(f"cos_sin_cache must be contiguous float32 (max_position, {head_dim})")
    if gamma is not None:
        _C.require_cuda(gamma)
        if gamma.dtype != torch.float32 or gamma.numel() != head_dim or not gamma.is_contiguous():
            raise ValueError(f"gamma must be contiguous float32 ({head_dim},)")
    int8 = False
    num_slots = 0
    if slot_mapping is not None:
        if k_cache is None or v_cache is None:
            raise ValueError("slot_mapping given without caches")
        _C.require_cuda(slot_mapping, k_cache, v_cache)
        if slot_mapping.numel() != num_tokens:
            raise ValueError("Slot mapping size must match number of tokens")
        if slot_mapping.dtype != torch.int64:
            slot_mapping = slot_mapping.to(torch.int64)
        slot_mapping = slot_mapping.contiguous()
        for name, c in (("k_cache", k_cache), ("v_cache", v_cache)):
            if c.dim() != 4 or tuple(c.shape[2:]) != (num_kv_heads, head_dim) or not c.is_contiguous():
                raise ValueError(f"{name} must be contiguous [num_blocks, block_size, {num_kv_heads}, {head_dim}]")
        if k_cache.shape != v_cache.shape:
            raise ValueError("K and V cache shapes must match")
        int8 = k_cache.dtype == torch.int8
        if int8:
            if v_cache.dtype != torch.int8:
                raise ValueError("int8 caches expected")
            for name, s in (("k_scale", k_scale), ("v_scale", v_scale)):
                if s is None or s.dtype != torch.float32 or tuple(s.shape) != tuple(k_cache.shape[:3]) \
                        or not s.is_contiguous():
                    raise ValueError(f"{name} must be contiguous float32 {tuple(k_cache.shape[:3])}")
        elif k_cache.dtype != q.dtype or v_cache.dtype != q.dtype:
            raise ValueError(f"cache dtype {k_cache.dtype} differs from q/k/v dtype {q.dtype}")
        num_slots = k_cache.shape[0] * k_cache.shape[1]
    q_out = torch.empty((num_tokens, num_heads, head_dim), dtype=q.dtype, device=q.device)
    k_out = torch.empty((num_tokens, num_kv_heads, head_dim), dtype=q.dtype, device=q.device) if need_kv else None
    v_out = torch.empty_like(k_out) if need_kv else None
    if num_tokens == 0:
        return q_out, k_out, v_out
    lib = _C.load()
    st = lib.mvllm_qk_norm_rope_store(
        _ptr(q_out), _ptr(k_out), _ptr(v_out), _ptr(q), _ptr(k), _ptr(v), q_stride, k_stride, v_stride,
        _ptr(gamma), float(eps), _ptr(cos_sin_cache), cos_sin_cache.shape[0], _ptr(positions),
        _ptr(slot_mapping), _ptr(k_cache), _ptr(v_cache), _ptr(k_scale if int8 else None),
        _ptr(v_scale if int8 else None), int(int8), num_tokens, num_slots, num_heads, num_kv_heads, head_dim,
        _C.dtype_code(q.dtype), _C.current_stream_ptr(q.device))
    _C.check(st, "qk_norm_rope_store")
    return q_out, k_out, v_out


def sample_tokens(logits: torch.Tensor, temperatures: torch.Tensor, seed: int = 0, offset: int = 0,
                  noise: torch.Tensor | None = None, use_workspace: bool = True) -> torch.Tensor:
    """One token per row from softmax(logits / temperature): argmax of ``probs / Exp(1) noise`` as in
    sampler.py:15-18, computed as argmax(logits / T - log(noise)) without a probability tensor.

    logits: (batch, vocab) float32 / bfloat16 / float16, rows may be strided; temperatures float32 (batch,), > 0.
    ``noise`` float32 (batch, vocab) supplies the draws (clamped below at 1e-10); without it they are generated
    from (seed, offset): the same pair always gives the same tokens, advance ``offset`` per call.
    ``use_workspace=False`` keeps every row in one workgroup (same tokens, slower for small batches).
    Returns int64 (batch,).
    """
    _C.require_cuda(logits, temperatures, noise)
    if logits.dim() != 2:
        raise ValueError(f"logits must be (batch, vocab), got {tuple(logits.shape)}")
    batch, vocab = logits.shape
    if batch > 1 and logits.stride(1) != 1 or batch == 1 and vocab > 1 and logits.stride(1) != 1:
        logits = logits.contiguous()
    if temperatures.numel() != batch:
        raise ValueError("temperatures must have one entry per row")
    temperatures = temperatures.to(torch.float32).contiguous()
    if noise is not None:
        if tuple(noise.shape) != (batch, vocab) or noise.dtype != torch.float32:
            raise ValueError(f"noise must be float32 ({batch}, {vocab})")
        noise = noise.contiguous()
    out = torch.empty(batch, dtype=torch.int64, device=logits.device)
    if batch == 0:
        return out
    lib = _C.load()
    nbytes = lib.mvllm_sample_tokens_workspace_bytes(batch, vocab) if use_workspace else 0
    ws = torch.empty(nbytes, dtype=torch.uint8, device=logits.device) if nbytes else None
    st = lib.mvllm_sample_tokens(_ptr(out), _ptr(logits), logits.stride(0) if batch > 1 else vocab,
                                 _ptr(temperatures), _ptr(noise), int(seed) & (2 ** 64 - 1),
                                 int(offset) & (2 ** 64 - 1), batch, vocab, _C.dtype_code(logits.dtype),
                                 _ptr(ws), nbytes, _C.current_stream_ptr(logits.device))
    _C.check(st, "sample_tokens")
    return out


def sample_tokens_into(out: torch.Tensor, logits: torch.Tensor, temperatures: torch.Tensor, seed: int,
                       offset_dev: torch.Tensor, workspace: torch.Tensor | None) -> None:
    """``sample_tokens`` for a captured graph: nothing is allocated (``out`` int64 (batch,), ``workspace`` uint8 from
    ``sample_workspace_bytes`` or None) and the call offset is read from ``offset_dev`` (one uint64 / int64 on the
    device, which the graph increments), so every replay draws fresh noise."""
    _C.require_cuda(out, logits, temperatures, offset_dev, workspace)
    batch, vocab = logits.shape
    if logits.stride(1) != 1 or out.numel() != batch or out.dtype != torch.int64 or temperatures.dtype != torch.float32:
        raise ValueError("logits rows must be dense, out int64 (batch,), temperatures float32 (batch,)")
    st = _C.load().mvllm_sample_tokens_dev_offset(
        _ptr(out), _ptr(logits), logits.stride(0) if batch > 1 else vocab, _ptr(temperatures),
        int(seed) & (2 ** 64 - 1), _ptr(offset_dev), batch, vocab, _C.dtype_code(logits.dtype), _ptr(workspace),
        0 if workspace is None else workspace.numel(), _C.current_stream_ptr(logits.device))
    _C.check(st, "sample_tokens_into")


def sample_workspace_bytes(batch: int, vocab: int) -> int:
    return int(_C.load().mvllm_sample_tokens_workspace_bytes(batch, vocab))


def decode_advance(input_ids: torch.Tensor, context_lens: torch.Tensor, positions: torch.Tensor,
                   slot_mapping: torch.Tensor, sampled: torch.Tensor, step: torch.Tensor | None = None,
                   host_ids: torch.Tensor | None = None) -> None:
    """Move a decode batch's step metadata one token forward on the device (all int64 (batch,), in place):
    input = the id sampled last step, context length + 1, position = new length - 1, slot + 1; rows whose context
    length is not positive (padding of a captured batch size) stay as they are.  ``step`` (one int64 / uint64 on the
    device): the sampler's call counter, incremented by one in the same launch.  ``host_ids`` (with ``step``): a
    pinned int64 CPU tensor (2, n >= batch + 1); row ``step & 1`` (before the increment) receives the sampled ids and
    then, in its last entry, the new counter value, written by the kernel itself: the host may read the ids as soon as
    it sees that value."""
    _C.require_cuda(input_ids, context_lens, positions, slot_mapping, sampled, step)
    n = sampled.numel()
    for t in (input_ids, context_lens, positions, slot_mapping, sampled):
        if t.dtype != torch.int64 or t.numel() < n or not t.is_contiguous():
            raise ValueError("decode_advance takes contiguous int64 tensors of at least the batch size")
    if step is not None and (step.numel() != 1 or step.element_size() != 8):
        raise ValueError("step must be one 64-bit integer on the device")
    host_ptr, host_stride = 0, 0
    if host_ids is not None:
        if step is None or host_ids.is_cuda or not host_ids.is_pinned() or host_ids.dtype != torch.int64 \
                or host_ids.dim() != 2 or host_ids.shape[0] != 2 or host_ids.shape[1] < n + 1 or not host_ids.is_contiguous():
            raise ValueError("host_ids must be a pinned contiguous int64 CPU tensor (2, >= batch + 1), given with step")
        host_ptr, host_stride = host_ids.data_ptr(), host_ids.shape[1]
    st = _C.load().mvllm_decode_advance(_ptr(input_ids), _ptr(context_lens), _ptr(positions), _ptr(slot_mapping),
                                        _ptr(sampled), _ptr(step), host_ptr, host_stride, n,
                                        _C.current_stream_ptr(sampled.device))
    _C.check(st, "decode_advance")


def _rows2d(name, t):
    if t.dim() != 2:
        raise ValueError(f"{name} must be (rows, features), got {tuple(t.shape)}")
    if t.shape[0] > 1 and t.stride(1) != 1 or t.shape[0] == 1 and t.shape[1] > 1 and t.stride(1) != 1:
        t = t.contiguous()
    return t, (t.stride(0) if t.shape[0] > 1 else t.shape[1])


def add_rms_norm(x: torch.Tensor, gamma: torch.Tensor, eps: float, residual: torch.Tensor | None = None):
    """``LayerNorm.forward`` (layers/layernorm.py:9-28) in one launch.

    Without ``residual``: returns ``x / sqrt(mean(x^2) + eps) * gamma``.  With it: returns
    ``(norm(x + residual), x + residual)``, the sum rounded to x's dtype first.  x, residual: (rows, hidden),
    rows may be strided; gamma float32 (hidden,).
    """
    _C.require_cuda(x, gamma, residual)
    x, x_stride = _rows2d("x", x)
    rows, hidden = x.shape
    if gamma.dtype != torch.float32 or gamma.numel() != hidden or not gamma.is_contiguous():
        raise ValueError(f"gamma must be contiguous float32 ({hidden},)")
    r_stride = hidden
    if residual is not None:
        if residual.shape != x.shape or residual.dtype != x.dtype:
            raise ValueError("residual must match x in shape and dtype")
        residual, r_stride = _rows2d("residual", residual)
    out = torch.empty((rows, hidden), dtype=x.dtype, device=x.device)
    new_residual = torch.empty_like(out) if residual is not None else None
    if rows:
        lib = _C.load()
        st = lib.mvllm_add_rms_norm(_ptr(out), _ptr(new_residual), _ptr(x), _ptr(residual), _ptr(gamma), float(eps),
                                    rows, hidden, x_stride, r_stride, _C.dtype_code(x.dtype),
                                    _C.current_stream_ptr(x.device))
        _C.check(st, "add_rms_norm")
    return out if residual is None else (out, new_residual)


def silu_and_mul(x: torch.Tensor) -> torch.Tensor:
    """``SiluAndMul.forward`` (layers/activation.py:15-18): silu(first half) * second half of the last dim."""
    _C.require_cuda(x)
    x, stride = _rows2d("x", x)
    rows, two_w = x.shape
    if two_w % 2:
        raise ValueError("the last dimension must be even")
    out = torch.empty((rows, two_w // 2), dtype=x.dtype, device=x.device)
    if rows:
        lib = _C.load()
        st = lib.mvllm_silu_and_mul(_ptr(out), _ptr(x), rows, two_w // 2, stride, _C.dtype_code(x.dtype),
                                    _C.current_stream_ptr(x.device))
        _C.check(st, "silu_and_mul")
    return out


def gated_unit(x: torch.Tensor, out: torch.Tensor | None = None, alpha: float = 1.0, limit: float = math.inf,
               shift: float = 0.0) -> torch.Tensor:
    """g sigmoid(alpha g) (u + shift) of the halves of x's rows, g at most ``limit`` and u within +-``limit``; rows of x and
    ``out`` may be strided.  By default silu(g) * u, rounded once."""
    _C.require_cuda(x, out)
    rows, width = x.shape[0], x.shape[1] // 2
    if x.dim() != 2 or x.shape[1] % 2 or x.stride(1) != 1:
        raise ValueError("x must be (rows, 2 * width) with dense rows")
    if out is None:
        out = torch.empty((rows, width), dtype=x.dtype, device=x.device)
    if tuple(out.shape) != (rows, width) or out.dtype != x.dtype or out.stride(1) != 1:
        raise ValueError(f"out must be ({rows}, {width}) in x's dtype with dense rows")
    st = _C.load().mvllm_gated_unit(_ptr(out), out.stride(0) if rows > 1 else width, _ptr(x), x.stride(0) if rows > 1 else 2 * width, rows,
                                    width, float(alpha), float(limit), float(shift), _C.dtype_code(x.dtype), _C.current_stream_ptr(x.device))
    _C.check(st, "gated_unit")
    return out


def gelu_tanh(x: torch.Tensor, out: torch.Tensor | None = None) -> torch.Tensor:
    """The tanh form of gelu of x's rows (strided; ``out`` may be x itself)."""
    _C.require_cuda(x, out)
    rows, width = x.shape
    out = torch.empty((rows, width), dtype=x.dtype, device=x.device) if out is None else out
    if tuple(out.shape) != (rows, width) or out.dtype != x.dtype or out.stride(1) != 1 or x.stride(1) != 1:
        raise ValueError(f"x and out must be ({rows}, {width}) in one dtype with dense rows")
    st = _C.load().mvllm_gelu_tanh(_ptr(out), out.stride(0) if rows > 1 else width, _ptr(x), x.stride(0) if rows > 1 else width, rows,
                                   width, _C.dtype_code(x.dtype), _C.current_stream_ptr(x.device))
    _C.check(st, "gelu_tanh")
    return out


def linear_small_m_takes(x: torch.Tensor, weight: torch.Tensor, max_rows: int = 64) -> bool:
    """Whether ``linear_small_m`` is built for this call: at most 64 rows, bf16 / fp16 on the GPU, N a multiple of 16,
    K a multiple of 512, rows of x dense."""
    return (x.is_cuda and x.dim() == 2 and 0 < x.shape[0] <= min(max_rows, 64) and x.dtype in (torch.bfloat16, torch.float16)
            and weight.dtype == x.dtype and weight.is_contiguous() and weight.shape[0] % 16 == 0
            and weight.shape[1] % 512 == 0 and x.stride(1) == 1 and x.stride(0) % 8 == 0
            and x.data_ptr() % 16 == 0)


def linear_small_m(x: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor | None = None, gelu: bool = False) -> torch.Tensor:
    """``F.linear(x, weight, bias)`` for the few rows of a decode step (the reference's projections,
    models/qwen3.py:90-94, 118, 121-160, are library GEMMs): one HIP launch in which every wave asks for its whole
    share of the weights at once, so the call costs about one memory round trip.  x (M <= 64, K), weight (N, K)
    contiguous, bias (N,) or None, all in one 16-bit dtype; fp32 accumulation.  ``gelu``: the result through the tanh form
    of gelu, rounded once.  Returns (M, N)."""
    _C.require_cuda(x, weight, bias)
    if x.dim() != 2 or weight.dim() != 2 or weight.shape[1] != x.shape[1]:
        raise ValueError(f"x (M, K) and weight (N, K) expected, got {tuple(x.shape)} and {tuple(weight.shape)}")
    if weight.dtype != x.dtype or (bias is not None and bias.dtype != x.dtype):
        raise ValueError("x, weight and bias must share one dtype")
    if not weight.is_contiguous() or x.stride(1) != 1:
        raise ValueError("weight must be contiguous and the rows of x dense")
    m, k = x.shape
    n = weight.shape[0]
    out = torch.empty(m, n, dtype=x.dtype, device=x.device)
    lib = _C.load()
    st = (lib.mvllm_linear_small_m_gelu if gelu else lib.mvllm_linear_small_m)(
        _ptr(out), _ptr(x), _ptr(weight), _ptr(bias), x.stride(0) if m > 1 else k, m, n, k, _C.dtype_code(x.dtype),
        _C.current_stream_ptr(x.device))
    _C.check(st, "linear_small_m")
    return out


_PLAN_CACHE: dict = {}


def norm_linear_small_m_takes(x: torch.Tensor, weight: torch.Tensor, max_rows: int = 32, norm: bool = True,
                              glu: bool = False) -> bool:
    """Whether ``norm_linear_small_m`` is built for this call (``mvllm_linear_small_m_plan``, remembered per shape)."""
    if not linear_small_m_takes(x, weight, max_rows) or not x.is_contiguous():
        return False
    key = (x.shape[0], weight.shape[0], weight.shape[1], norm, glu, x.dtype)
    if key not in _PLAN_CACHE:
        st = _C.load().mvllm_linear_small_m_plan(key[0], key[1], key[2], int(norm), int(glu), _C.dtype_code(x.dtype), None)
        _PLAN_CACHE[key] = st == 0
    return _PLAN_CACHE[key]


def norm_linear_small_m(x: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor | None = None,
                        gamma: torch.Tensor | None = None, eps: float = 1e-6, residual: torch.Tensor | None = None,
                        want_residual: bool = False, glu: bool = False):
    """A decode step's projection with the launches around it folded in (the reference runs them as separate
    modules, models/qwen3.py:151-160, 197-212): with ``gamma`` (float32, (K,)) the rows are first replaced by
    ``rms_norm(x + residual) * gamma`` as ``add_rms_norm`` computes it; with ``glu`` the weight is (2F, K) and the
    result ``silu(gate) * up`` as ``silu_and_mul`` computes it.  Returns the (M, N) or (M, F) product, and with
    ``want_residual`` also ``x + residual`` in x's dtype (a new tensor)."""
    _C.require_cuda(x, weight, bias, gamma, residual)
    if x.dim() != 2 or weight.dim() != 2 or weight.shape[1] != x.shape[1]:
        raise ValueError(f"x (M, K) and weight (N, K) expected, got {tuple(x.shape)} and {tuple(weight.shape)}")
    if weight.dtype != x.dtype or (bias is not None and bias.dtype != x.dtype) or (residual is not None and residual.dtype != x.dtype):
        raise ValueError("x, weight, bias and residual must share one dtype")
    if not weight.is_contiguous() or x.stride(1) != 1:
        raise ValueError("weight must be contiguous and the rows of x dense")
    m, k = x.shape
    n = weight.shape[0]
    if gamma is not None and (gamma.dtype != torch.float32 or tuple(gamma.shape) != (k,)):
        raise ValueError("gamma must be float32 of shape (K,)")
    if residual is not None and (tuple(residual.shape) != (m, k) or not residual.is_contiguous()):
        raise ValueError("residual must be a contiguous (M, K) tensor")
    if (residual is not None or want_residual) and gamma is None:
        raise ValueError("a residual needs the norm (gamma)")
    out = torch.empty(m, n // 2 if glu else n, dtype=x.dtype, device=x.device)
    res_out = torch.empty(m, k, dtype=x.dtype, device=x.device) if want_residual else None
    st = _C.load().mvllm_norm_linear_small_m(_ptr(out), _ptr(res_out), _ptr(x), _ptr(residual), _ptr(gamma), float(eps),
                                             _ptr(weight), _ptr(bias), x.stride(0) if m > 1 else k, m, n, k, int(glu),
                                             _C.dtype_code(x.dtype), _C.current_stream_ptr(x.device))
    _C.check(st, "norm_linear_small_m")
    return (out, res_out) if want_residual else out


def lm_head_sample_takes(hidden: torch.Tensor, weight: torch.Tensor, batch: int | None = None) -> bool:
    """Whether ``lm_head_sample`` is built for this call: at most 64 rows to sample, bf16 / fp16 on the GPU, a
    vocabulary that is a multiple of 16, hidden size 256, 512 or 1024."""
    rows = hidden.shape[0] if batch is None else batch
    return (hidden.is_cuda and hidden.dim() == 2 and 0 < rows <= 64 and hidden.dtype in (torch.bfloat16, torch.float16)
            and weight.dtype == hidden.dtype and weight.dim() == 2 and weight.is_contiguous()
            and weight.shape[0] % 16 == 0 and weight.shape[1] in (256, 512, 1024) and hidden.shape[1] == weight.shape[1]
            and hidden.stride(1) == 1 and hidden.stride(0) % 8 == 0 and hidden.data_ptr() % 16 == 0)


def lm_head_sample_workspace_bytes(batch: int, hidden_size: int) -> int:
    return int(_C.load().mvllm_lm_head_sample_workspace_bytes(batch, hidden_size))


def lm_head_sample(hidden: torch.Tensor, weight: torch.Tensor, temperatures: torch.Tensor, seed: int = 0,
                   offset: int = 0, row_index: torch.Tensor | None = None, out: torch.Tensor | None = None,
                   offset_dev: torch.Tensor | None = None, workspace: torch.Tensor | None = None) -> torch.Tensor:
    """The LM head and the sampler in one pass over ``weight`` (vocab, K): the reference's
    ``ParallelLMHead.forward`` (layers/embedding_head.py:56-77) and ``SamplerLayer.forward`` (layers/sampler.py:14-19)
    without the (batch, vocab) logits.  Row ``b`` samples from ``hidden[row_index[b]]`` (``row_index`` None: row b) at
    ``temperatures[b]``; the noise is the in-kernel Philox stream of ``sample_tokens`` (same seed / offset: the same
    ids as ``sample_tokens(F.linear(hidden, weight), ...)`` up to the summation order inside a logit).  ``out``,
    ``offset_dev`` and ``workspace`` (uint8, ``lm_head_sample_workspace_bytes``) let a captured graph call it without
    allocating and draw fresh noise on every replay."""
    _C.require_cuda(hidden, weight, temperatures, row_index, out, offset_dev, workspace)
    batch = hidden.shape[0] if row_index is None else row_index.numel()
    if not lm_head_sample_takes(hidden, weight, batch):
        raise ValueError("lm_head_sample: shape or dtype not taken (see lm_head_sample_takes)")
    if temperatures.dtype != torch.float32 or temperatures.numel() != batch or not temperatures.is_contiguous():
        raise ValueError("temperatures must be contiguous float32 (batch,)")
    if row_index is not None and (row_index.dtype != torch.int64 or not row_index.is_contiguous()):
        raise ValueError("row_index must be contiguous int64")
    vocab, k = weight.shape
    if out is None:
        out = torch.empty(batch, dtype=torch.int64, device=hidden.device)
    elif out.dtype != torch.int64 or out.numel() != batch or not out.is_contiguous():
        raise ValueError("out must be contiguous int64 (batch,)")
    need = lm_head_sample_workspace_bytes(batch, k)
    if workspace is None:
        workspace = torch.empty(need, dtype=torch.uint8, device=hidden.device)
    st = _C.load().mvllm_lm_head_sample(_ptr(out), _ptr(hidden), hidden.stride(0) if hidden.shape[0] > 1 else k,
                                        _ptr(row_index), _ptr(weight), _ptr(temperatures), int(seed) & (2 ** 64 - 1),
                                        int(offset) & (2 ** 64 - 1), _ptr(offset_dev), batch, vocab, k,
                                        _C.dtype_code(hidden.dtype), _ptr(workspace), workspace.numel(),
                                        _C.current_stream_ptr(hidden.device))
    _C.check(st, "lm_head_sample")
    return out


def _check(t, dtype, shape, name):
    if t.dtype != dtype or tuple(t.shape) != tuple(shape) or not t.is_contiguous():
        raise ValueError(f"{name} must be contiguous {dtype} {tuple(shape)}, got {t.dtype} {tuple(t.shape)}")


def norm_conv(step, pre: torch.Tensor, eps: float, dtype: torch.dtype, x: torch.Tensor | None = None,
              tokens: torch.Tensor | None = None, embed: torch.Tensor | None = None, y: torch.Tensor | None = None,
              post: torch.Tensor | None = None, conv: torch.Tensor | None = None, state: torch.Tensor | None = None,
              want_x: bool = True):
    """The launch between two sublayers: ``x' = x + rms(y) * post``, ``h = rms(x') * pre``, ``h + conv(h)`` over time.

    x float32 (T, W), or ``embed`` (vocab, W) with ``tokens`` int64 (T,); y (T, W) in ``dtype`` or None; post / pre
    float32 gains, one number () or per channel (W,); conv float32 (taps, W) or None with ``state`` float32
    (banks, taps - 1, W); ``step``: the ragged step (entries, banks, positions).  Returns (out in ``dtype``, x')."""
    _C.require_cuda(pre, x, tokens, embed, y, post, conv, state)
    src = x if x is not None else embed
    rows, width = (x.shape[0] if x is not None else tokens.numel()), src.shape[1]
    if x is not None:
        _check(x, torch.float32, (rows, width), "x")
    else:
        _check(embed, dtype, embed.shape, "embed")
        _check(tokens, torch.int64, (rows,), "tokens")
    if y is not None:
        _check(y, dtype, (rows, width), "y")
    for name, g in (("pre", pre), ("post", post)):
        if g is not None and (g.dtype != torch.float32 or g.numel() not in (1, width) or not g.is_contiguous()):
            raise ValueError(f"{name} must be float32, one number or ({width},)")
    taps = banks = 0
    if conv is not None:
        taps = conv.shape[0]
        _check(conv, torch.float32, (taps, width), "conv")
        if taps > 1:
            banks = state.shape[0]
            _check(state, torch.float32, (banks, taps - 1, width), "state")
        banks = max(banks, 1)
        if step.num_tokens != rows:
            raise ValueError("the step's rows and x's differ")
    out = torch.empty((rows, width), dtype=dtype, device=src.device)
    x_out = torch.empty((rows, width), dtype=torch.float32, device=src.device) if want_x and (y is not None or x is None) else None
    st = _C.load().mvllm_norm_conv(
        _ptr(out), _ptr(x_out), _ptr(x), _ptr(embed if x is None else None), _ptr(tokens if x is None else None),
        0 if embed is None else embed.shape[0], _ptr(y), _ptr(post if y is not None else None),
        int(post is not None and post.numel() > 1), _ptr(pre), int(pre.numel() > 1), float(eps), _ptr(conv), taps,
        _ptr(state if taps > 1 else None), banks, _ptr(step.cu_seqlens if taps else None),
        _ptr(step.row_entry if taps else None), _ptr(step.bank_in if taps else None), _ptr(step.bank_out if taps else None),
        _ptr(step.positions if taps else None), rows, width, _C.dtype_code(dtype), _C.current_stream_ptr(src.device))
    _C.check(st, "norm_conv")
    return out, (x_out if x_out is not None else x)


def head_rope_store(proj: torch.Tensor, positions: torch.Tensor, num_heads: int, num_kv_heads: int, dim: int, vdim: int,
                    head_dim: int, gain_q: torch.Tensor | None = None, gain_k: torch.Tensor | None = None,
                    eps: float = 1e-6, q_scale: float = 1.0, rot_table: torch.Tensor | None = None,
                    v_table: torch.Tensor | None = None, interleaved: bool = True, dst_row: torch.Tensor | None = None,
                    slots: torch.Tensor | None = None, k_cache: torch.Tensor | None = None,
                    v_cache: torch.Tensor | None = None, need_kv: bool = True, row_norm: bool = False, unit_qk: bool = False,
                    unit_v: bool = False, head_scale: torch.Tensor | None = None, kv_cache: torch.Tensor | None = None,
                    kv_out: torch.Tensor | None = None, kv_rows: torch.Tensor | None = None):
    """Norms, rotary embedding, rotated values and the cache store of packed projection rows [q | k | v | ...].

    ``rot_table`` float32 (max_position, rot_dims / 2, 2) and ``v_table`` (max_position, vdim / 2, 2) hold (cos, sin) per
    pair; ``interleaved`` pairs dims 2i and 2i + 1, otherwise the halves.  Heads leave ``head_dim`` wide, zeros past
    ``dim`` / ``vdim``; row t goes to row ``dst_row[t]`` of the packed results.  Gains norm every head, with ``row_norm`` all
    heads of a row at once (gains of that many numbers); ``unit_qk`` / ``unit_v``: every head of q and k behind the rotation /
    of v over its root mean square; ``head_scale`` float32 (num_heads,): a further factor of q.  Returns (q, k, v), k and v None
    unless ``need_kv``.

    With ``kv_cache`` (blocks, block_size, num_kv_heads, 2 head_dim) a key and its value are neighbours; ``kv_out`` (n,
    num_kv_heads, 2 head_dim) takes them packed at rows ``kv_rows`` int64 (negative: none; None: t).  Returns q."""
    _C.require_cuda(proj, positions, gain_q, gain_k, rot_table, v_table, dst_row, slots, k_cache, v_cache, head_scale, kv_cache,
                    kv_out, kv_rows)
    rows = proj.shape[0]
    if proj.dim() != 2 or (proj.shape[1] > 1 and proj.stride(1) != 1) or proj.shape[1] < num_heads * dim + num_kv_heads * (dim + vdim):
        raise ValueError("proj must be (T, >= q + k + v columns) with dense rows")
    _check(positions, torch.int64, (rows,), "positions")
    for name, g in (("gain_q", gain_q), ("gain_k", gain_k)):
        if g is not None:
            _check(g, torch.float32, (dim * (1 if not row_norm else num_heads if name == "gain_q" else num_kv_heads),), name)
    if head_scale is not None:
        _check(head_scale, torch.float32, (num_heads,), "head_scale")
    tables = [t for t in (rot_table, v_table) if t is not None]
    max_position = min((t.shape[0] for t in tables), default=1 << 62)
    rot = 0 if rot_table is None else 2 * rot_table.shape[1]
    for name, t, n in (("rot_table", rot_table, rot // 2), ("v_table", v_table, vdim // 2)):
        if t is not None:
            _check(t, torch.float32, (t.shape[0], n, 2), name)
    if dst_row is not None:
        _check(dst_row, torch.int32, (rows,), "dst_row")
    num_slots = 0
    if slots is not None:
        _check(slots, torch.int64, (rows,), "slots")
        for name, c, d in (("kv_cache", kv_cache, 2 * head_dim),) if kv_cache is not None else (
                ("k_cache", k_cache, head_dim), ("v_cache", v_cache, head_dim)):
            _check(c, proj.dtype, (*c.shape[:2], num_kv_heads, d), name)
            num_slots = min(num_slots or c.shape[0] * c.shape[1], c.shape[0] * c.shape[1])
    q = torch.empty((rows, num_heads, head_dim), dtype=proj.dtype, device=proj.device)
    k = v = None
    behind = head_dim * proj.element_size()
    if kv_cache is not None:
        caches = (kv_cache.data_ptr(), kv_cache.data_ptr() + behind) if slots is not None else (0, 0)
        packed = (0, 0)
        if kv_out is not None:
            _check(kv_out, proj.dtype, (kv_out.shape[0], num_kv_heads, 2 * head_dim), "kv_out")
            if kv_rows is None and kv_out.shape[0] < rows:
                raise ValueError("kv_out has fewer rows than proj")
            packed = (kv_out.data_ptr(), kv_out.data_ptr() + behind)
        if kv_rows is not None:
            _check(kv_rows, torch.int64, (rows,), "kv_rows")
        if dst_row is not None:
            raise ValueError("kv_rows instead of dst_row")
    else:
        if need_kv:
            k = torch.empty((rows, num_kv_heads, head_dim), dtype=proj.dtype, device=proj.device)
            v = torch.empty_like(k)
        caches = (_ptr(k_cache), _ptr(v_cache)) if slots is not None else (0, 0)
        packed, kv_rows = (_ptr(k), _ptr(v)), None
    st = _C.load().mvllm_head_norm_rope_store(
        _ptr(q), *packed, _ptr(kv_rows), _ptr(proj), proj.stride(0) if rows > 1 else proj.shape[1], _ptr(gain_q), _ptr(gain_k),
        int(row_norm) + 2 * int(unit_qk) + 4 * int(unit_v), float(eps), float(q_scale), _ptr(head_scale), _ptr(rot_table), rot,
        _ptr(v_table), int(interleaved), max_position, _ptr(positions), _ptr(dst_row), _ptr(slots), *caches,
        head_dim * (1 if kv_cache is None else 2), num_slots, rows, num_heads, num_kv_heads, dim, vdim, head_dim,
        _C.dtype_code(proj.dtype), _C.current_stream_ptr(proj.device))
    _C.check(st, "head_rope_store")
    return q if kv_cache is not None else (q, k, v)


def head_unrotate_gate(o: torch.Tensor, positions: torch.Tensor, vdim: int, gate: torch.Tensor | None = None,
                       v_table: torch.Tensor | None = None, interleaved: bool = True,
                       dst_row: torch.Tensor | None = None) -> torch.Tensor:
    """``o`` (T, heads, head_dim) from attention over rotated values -> (T, heads * vdim): every head turned back by its
    position (``v_table`` None: not) and multiplied by ``sigmoid(gate)``, gate (T, heads) with dense rows or None; row t is
    read from row ``dst_row[t]``."""
    _C.require_cuda(o, positions, gate, v_table, dst_row)
    rows, heads, head_dim = o.shape
    _check(o, o.dtype, (rows, heads, head_dim), "o")
    _check(positions, torch.int64, (rows,), "positions")
    if gate is not None and (gate.dtype != o.dtype or tuple(gate.shape) != (rows, heads) or (heads > 1 and gate.stride(1) != 1)):
        raise ValueError("gate must be (T, heads) in o's dtype with dense rows")
    if v_table is not None:
        _check(v_table, torch.float32, (v_table.shape[0], vdim // 2, 2), "v_table")
    if dst_row is not None:
        _check(dst_row, torch.int32, (rows,), "dst_row")
    out = torch.empty((rows, heads * vdim), dtype=o.dtype, device=o.device)
    st = _C.load().mvllm_head_unrotate_gate(
        _ptr(out), _ptr(o), _ptr(gate), heads if gate is None or rows == 1 else gate.stride(0), _ptr(v_table), int(interleaved),
        1 << 62 if v_table is None else v_table.shape[0], _ptr(positions), _ptr(dst_row), rows, heads, vdim, head_dim,
        _C.dtype_code(o.dtype), _C.current_stream_ptr(o.device))
    _C.check(st, "head_unrotate_gate")
    return out


def chunk_decode_step(context_lens: torch.Tensor, block_tables: torch.Tensor, chunk: int, block_size: int,
                      chunk_lens: torch.Tensor, slots: torch.Tensor) -> None:
    """Per row of a decode batch over a cache that holds one attention chunk per sequence (``chunk`` 0: all of it): the
    context length inside the chunk and the cache slot of the row's token, written to ``chunk_lens`` and ``slots`` (int64,
    in place); 0 and -1 for rows whose context length is 0."""
    _C.require_cuda(context_lens, block_tables, chunk_lens, slots)
    batch = context_lens.numel()
    for name, t in (("context_lens", context_lens), ("chunk_lens", chunk_lens), ("slots", slots)):
        _check(t, torch.int64, (batch,), name)
    _check(block_tables, torch.int32, (batch, block_tables.shape[1]), "block_tables")
    st = _C.load().mvllm_chunk_decode_step(_ptr(chunk_lens), _ptr(slots), _ptr(context_lens), _ptr(block_tables),
                                           block_tables.shape[1], int(chunk), block_size, batch,
                                           _C.current_stream_ptr(context_lens.device))
    _C.check(st, "chunk_decode_step")


def _stream_weights(streams, hc_in, hc_out=None, hc_mix=None):
    for name, t, shape in (("hc_in", hc_in, (streams,)), ("hc_out", hc_out, (streams,)), ("hc_mix", hc_mix, (streams, streams))):
        if t is not None:
            _check(t, torch.float32, shape, name)


def stream_embed_norm(step, tokens: torch.Tensor, embed: torch.Tensor, scale: float, streams: int, gain: torch.Tensor, eps: float,
                      hc_in: torch.Tensor | None = None, bigram: torch.Tensor | None = None, hashing: tuple = (1, 0, 0),
                      prev_tokens: torch.Tensor | None = None, padded: int = 0):
    """The front of a model with several residual streams: every stream starts as ``embed[token] * scale`` plus, with
    ``bigram`` (buckets + 1, W), the row (previous token * mul_prev + token * mul_cur) mod buckets of it, ``hashing`` =
    (buckets, mul_prev, mul_cur); a sequence's first token has row ``buckets``.  ``prev_tokens`` int64 (banks,) is the part of
    a sequence's state that holds the token before a step's first.

    Returns (rms(sum_s hc_in[s] x_s) * gain, filled up with zeros to ``padded`` columns, in embed's dtype; x float32
    (T, streams, W))."""
    _C.require_cuda(tokens, embed, gain, hc_in, bigram, prev_tokens)
    rows, width = tokens.numel(), embed.shape[1]
    padded = max(padded, width)
    _check(tokens, torch.int64, (rows,), "tokens")
    _check(embed, embed.dtype, embed.shape, "embed")
    _check(gain, torch.float32, (width,), "gain")
    _stream_weights(streams, hc_in)
    if step.num_tokens != rows:
        raise ValueError("the step's rows and the tokens differ")
    if bigram is not None:
        _check(bigram, embed.dtype, (hashing[0] + 1, width), "bigram")
        _check(prev_tokens, torch.int64, prev_tokens.shape, "prev_tokens")
    out = torch.empty((rows, padded), dtype=embed.dtype, device=embed.device)
    x = torch.empty((rows, streams, width), dtype=torch.float32, device=embed.device)
    st = _C.load().mvllm_stream_embed_norm(
        _ptr(out), padded, _ptr(x), _ptr(embed), embed.shape[0], float(scale), _ptr(bigram), *(int(n) for n in hashing),
        _ptr(prev_tokens), _ptr(tokens), _ptr(step.positions), _ptr(step.cu_seqlens), _ptr(step.row_entry), _ptr(step.bank_in),
        _ptr(step.bank_out), _ptr(hc_in), _ptr(gain), float(eps), rows, streams, width, _C.dtype_code(embed.dtype),
        _C.current_stream_ptr(embed.device))
    _C.check(st, "stream_embed_norm")
    return out, x


def stream_norm(x: torch.Tensor, y, hc_out: torch.Tensor, hc_mix: torch.Tensor, gain: torch.Tensor, eps: float,
                hc_in: torch.Tensor | None = None, scale: torch.Tensor | None = None, padded: int = 0, want_x: bool = True,
                dtype: torch.dtype | None = None):
    """A sublayer's result into the residual streams and the norm in front of the next one, in one launch:
    ``x_t <- sum_s hc_mix[s, t] x_s + hc_out[t] * scale * y`` for all streams at once, in place (``want_x`` False: not kept),
    then ``rms(sum_t hc_in[t] x_t) * gain`` (``hc_in`` None: the plain sum) with zeros up to ``padded`` columns.

    x float32 (T, streams, W); y (T, >= W) with dense rows, or a mixture's unsummed results (``layers.experts.ExpertOutput``);
    everything else float32.  Returns (the norm, x)."""
    parts = part_row = weights = gate = ids = own = None
    if not isinstance(y, torch.Tensor):
        parts, part_row, weights, gate, ids, own, y = y.parts, y.part_row, y.weights, y.gate, y.ids, y.inputs, y.shared
    _C.require_cuda(x, y, parts, part_row, weights, gate, ids, own, hc_out, hc_mix, gain, hc_in, scale)
    rows, streams, width = x.shape
    padded = max(padded, width)
    _check(x, torch.float32, (rows, streams, width), "x")
    _check(gain, torch.float32, (width,), "gain")
    _stream_weights(streams, hc_in, hc_out, hc_mix)
    if scale is not None:
        _check(scale, torch.float32, (width,), "scale")
    dtype = dtype or (y if y is not None else parts).dtype
    for name, t in (("y", y), ("parts", parts)):
        if t is not None and (t.dim() != 2 or t.dtype != dtype or t.shape[1] < width or t.stride(1) != 1):
            raise ValueError(f"{name} must be (*, >= {width}) in {dtype} with dense rows")
    if y is not None and y.shape[0] != rows:
        raise ValueError("y must have one row per row of x")
    top = 0
    if parts is not None:
        top = weights.shape[1]
        _check(weights, torch.float32, (rows, top), "weights")
        if parts.shape[0] != rows * top or (part_row is not None and (part_row.dtype != torch.int32 or part_row.numel() != rows * top
                                                                      or not part_row.is_contiguous())):
            raise ValueError("parts and part_row must have one row per choice")
        if gate is not None and (gate.dtype != torch.float32 or gate.numel() != rows):
            raise ValueError("gate must be float32, one number per row")
        if ids is not None:
            _check(ids, torch.int32, (rows, top), "ids")
            if own.dtype != dtype or own.dim() != 2 or own.shape[0] != rows or own.shape[1] < width or own.stride(1) != 1:
                raise ValueError(f"inputs must be ({rows}, >= {width}) in {dtype} with dense rows")
    out = torch.empty((rows, padded), dtype=dtype, device=x.device)
    st = _C.load().mvllm_stream_norm_identity(
        _ptr(out), padded, _ptr(x if want_x else None), _ptr(x), _ptr(y), 0 if y is None else max(y.stride(0), width), _ptr(parts),
        0 if parts is None else max(parts.stride(0), width), _ptr(part_row), _ptr(weights), top, _ptr(ids),
        _ptr(own), 0 if own is None else max(own.stride(0), width), _ptr(gate), 1 if gate is None else max(gate.stride(0), 1), _ptr(scale), _ptr(hc_out), _ptr(hc_mix), _ptr(hc_in), _ptr(gain), float(eps),
        rows, streams, width, _C.dtype_code(dtype), _C.current_stream_ptr(x.device))
    _C.check(st, "stream_norm")
    return out, x


def embed_rows(tokens: torch.Tensor, embed: torch.Tensor, scale: float, padded: int = 0):
    """The front of a model whose sublayers read the residual itself: (embed[token] * scale in embed's dtype, zeros up to
    ``padded`` columns; the same in float32)."""
    _C.require_cuda(tokens, embed)
    rows, width = tokens.numel(), embed.shape[1]
    padded = max(padded, width)
    _check(tokens, torch.int64, (rows,), "tokens")
    _check(embed, embed.dtype, embed.shape, "embed")
    out = torch.empty((rows, padded), dtype=embed.dtype, device=embed.device)
    x = torch.empty((rows, width), dtype=torch.float32, device=embed.device)
    st = _C.load().mvllm_embed_rows(_ptr(out), padded, _ptr(x), _ptr(embed), embed.shape[0], float(scale), _ptr(tokens), rows, width,
                                    _C.dtype_code(embed.dtype), _C.current_stream_ptr(embed.device))
    _C.check(st, "embed_rows")
    return out, x


def post_norm(x: torch.Tensor, y: torch.Tensor, gain: torch.Tensor, eps: float, centred: bool = True,
              final_gain: torch.Tensor | None = None, padded: int = 0, want_x: bool = True):
    """``x + norm(y) * gain`` into x (float32 (T, W), in place unless ``want_x`` is False), norm with the mean taken off
    (``centred``) or not.  Returns (what is read next, x): the new x in y's dtype with zeros up to ``padded`` columns, or with
    ``final_gain`` its norm times that."""
    _C.require_cuda(x, y, gain, final_gain)
    rows, width = x.shape
    padded = max(padded, width)
    _check(x, torch.float32, (rows, width), "x")
    for name, g in (("gain", gain), ("final_gain", final_gain)):
        if g is not None:
            _check(g, torch.float32, (width,), name)
    if y.dim() != 2 or y.shape[0] != rows or y.shape[1] < width or y.stride(1) != 1:
        raise ValueError(f"y must be ({rows}, >= {width}) with dense rows")
    out = torch.empty((rows, padded), dtype=y.dtype, device=y.device)
    st = _C.load().mvllm_post_norm(_ptr(out), padded, _ptr(x if want_x else None), _ptr(x), _ptr(y), max(y.stride(0), width), _ptr(gain),
                                   _ptr(final_gain), float(eps), int(centred), rows, width, _C.dtype_code(y.dtype),
                                   _C.current_stream_ptr(y.device))
    _C.check(st, "post_norm")
    return out, x
