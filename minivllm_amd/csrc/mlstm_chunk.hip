// The mLSTM recurrence of mlstm.hip in blocks of 64 rows on the matrix unit (memory_chunk.h).
#include "memory_chunk.h"

using namespace mvllm;

static int64_t chunk_ws_floats(int num_segments, int num_heads, int dim, int vdim) {
  return (int64_t)num_segments * num_heads * ((int64_t)dim * vdim + dim + 2) + 16;
}

extern "C" size_t mvllm_mlstm_chunked_workspace_bytes(int num_segments, int num_heads, int dim, int vdim) {
  if (num_segments <= 0 || num_heads <= 0 || dim <= 0 || vdim <= 0) return 0;
  return (size_t)chunk_ws_floats(num_segments, num_heads, dim, vdim) * sizeof(float);
}

extern "C" int mvllm_mlstm_chunked(float* num, float* den, float* m_next, const void* proj, int64_t proj_row_stride,
                                   const float* gates, float* s_state, float* n_state, const float* m_state,
                                   const int32_t* cu_seqlens, const int32_t* slots, const int64_t* positions,
                                   const int32_t* segments, int num_segments, int split, int num_heads, int dim, int vdim,
                                   float q_scale, float floor, int dtype, void* workspace, size_t workspace_bytes,
                                   void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (num_segments < 0 || num_heads <= 0 || dim <= 0 || vdim <= 0 || proj_row_stride < (int64_t)num_heads * (2 * dim + vdim))
    return MVLLM_ERR_BAD_SHAPE;
  if (dtype != MVLLM_BF16 || dim % 8 != 0 || vdim % 8 != 0 || proj_row_stride % 8 != 0 || dim > 256 || num_heads > 65535 ||
      proj_row_stride > (1 << 24) || vdim > (1 << 20) || (int64_t)num_heads * vdim > (1 << 22))
    return MVLLM_ERR_UNSUPPORTED;
  if (num_segments == 0) return MVLLM_OK;
  if (!num || !den || !m_next || !proj || !gates || !s_state || !n_state || !m_state || !cu_seqlens || !slots || !positions || !segments)
    return MVLLM_ERR_NULL_POINTER;
  if (!aligned16(proj)) return MVLLM_ERR_MISALIGNED;
  if (split && (!workspace || workspace_bytes < mvllm_mlstm_chunked_workspace_bytes(num_segments, num_heads, dim, vdim)))
    return MVLLM_ERR_WORKSPACE;
  if (split && (!aligned16(workspace) || !aligned16(s_state) || !aligned16(n_state))) return MVLLM_ERR_MISALIGNED;
  MemoryChunkArgs a = {};
  a.num = num; a.den = den; a.m_next = m_next; a.proj = reinterpret_cast<const bf16_t*>(proj); a.gates = gates;
  a.s_state = s_state; a.n_state = n_state; a.m_state = m_state; a.cu = cu_seqlens; a.slot = slots; a.positions = positions;
  a.segments = segments; a.proj_stride = proj_row_stride; a.num_segments = num_segments; a.heads = num_heads; a.dim = dim;
  a.vdim = vdim; a.q_scale = q_scale; a.floor = floor;
  const int64_t units = (int64_t)num_segments * num_heads;
  a.ws_s = reinterpret_cast<float*>(workspace);
  a.ws_n = split ? a.ws_s + units * dim * vdim : nullptr;
  a.ws_m = split ? a.ws_n + units * dim : nullptr;
  a.ws_f = split ? a.ws_m + units : nullptr;
  hipStream_t s = (hipStream_t)stream;
  return launch_chunked_sizes<true>(a, split != 0, s);
}
