// Matrix memory with a constant decay per head (lightning attention):
//     S = decay S + k v^T,  o = S^T q          (S [dim, vdim] per head and sequence, fp32; q, k, v optionally through silu)
// followed by one norm over all heads of a row and a gate per channel:
//     out = rms(o over the row) * weight * sigmoid(gate)
// mvllm_decay_memory_recurrent runs row by row (memory_recurrent.h: decoded tokens, short portions, fp32),
// mvllm_decay_memory_chunked in blocks of 64 rows on the matrix unit (memory_chunk.h), mvllm_gated_row_norm what follows.
#include "memory_chunk.h"
#include "memory_recurrent.h"
#include "row_sums.h"

namespace mvllm {

struct GatedNormArgs {
  void* out;               // [T, out_stride], zeros past the width
  const float* x;          // [T, W]
  const float* weight;     // [W]
  const void* gate;        // [T, gate_stride]
  int64_t out_stride, gate_stride;
  float eps;
  int width;
};

// One workgroup per row.
template <typename T, int VEC, int NC>
__global__ __launch_bounds__(kMaxThreads) void gated_row_norm_kernel(const GatedNormArgs a) {
  __shared__ float lds[2 * (kMaxThreads / 16)];
  const int64_t row = blockIdx.x;
  const int W = a.width, tid = threadIdx.x;
  const float* x_row = a.x + row * W;
  const T* g_row = reinterpret_cast<const T*>(a.gate) + row * a.gate_stride;
  T* out = reinterpret_cast<T*>(a.out) + row * a.out_stride;
  float x[NC][VEC], g[NC][VEC], w[NC][VEC], ss = 0.f;
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int at = (tid + c * blockDim.x) * VEC;
#pragma unroll
    for (int i = 0; i < VEC; ++i) x[c][i] = g[c][i] = w[c][i] = 0.f;
    if (at < W) {
      Chunk<float, VEC>::load(x_row + at, x[c]);
      Chunk<T, VEC>::load(g_row + at, g[c]);
      Chunk<float, VEC>::load(a.weight + at, w[c]);
    }
  }
#pragma unroll
  for (int c = 0; c < NC; ++c)
#pragma unroll
    for (int i = 0; i < VEC; ++i) ss = fmaf(x[c][i], x[c][i], ss);
  int flip = 0;
  block_sums<1>(&ss, lds, blockDim.x >> 6, flip);
  const float inv = 1.0f / sqrtf(ss / (float)W + a.eps);
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int at = (tid + c * blockDim.x) * VEC;
    if (at >= W) continue;
    float o[VEC];
#pragma unroll
    for (int i = 0; i < VEC; ++i) o[i] = x[c][i] * inv * w[c][i] / (1.0f + __expf(-g[c][i]));
    Chunk<T, VEC>::store(out + at, o);
  }
  for (int64_t c = W + tid; c < a.out_stride; c += blockDim.x) out[c] = from_float<T>(0.f);
}

template <typename T>
static int launch_gated_norm(const GatedNormArgs& a, int rows, hipStream_t s) {
  const uintptr_t mask = 4 * sizeof(T) - 1;
  const bool vec = a.width % 4 == 0 && a.gate_stride % 4 == 0 && a.out_stride % 4 == 0 && aligned16(a.x) && aligned16(a.weight) &&
                   (reinterpret_cast<uintptr_t>(a.gate) & mask) == 0 && (reinterpret_cast<uintptr_t>(a.out) & mask) == 0;
  const int chunks = vec ? a.width / 4 : a.width;
  int threads = min(rows <= 512 ? kMaxThreads : 256, (chunks + 63) / 64 * 64);
  int nc = (chunks + threads - 1) / threads;
  if (nc > 4) {
    threads = kMaxThreads;
    nc = (chunks + threads - 1) / threads;
  }
  if (nc > 8) return MVLLM_ERR_UNSUPPORTED;
  const dim3 grid((unsigned)rows), block((unsigned)threads);
  if (!vec) gated_row_norm_kernel<T, 1, 8><<<grid, block, 0, s>>>(a);
  else if (nc == 1) gated_row_norm_kernel<T, 4, 1><<<grid, block, 0, s>>>(a);
  else if (nc == 2) gated_row_norm_kernel<T, 4, 2><<<grid, block, 0, s>>>(a);
  else if (nc <= 4) gated_row_norm_kernel<T, 4, 4><<<grid, block, 0, s>>>(a);
  else gated_row_norm_kernel<T, 4, 8><<<grid, block, 0, s>>>(a);
  return launch_status();
}

}  // namespace mvllm

using namespace mvllm;

extern "C" int mvllm_decay_memory_recurrent(float* num, const void* proj, int64_t proj_row_stride, const float* decay,
                                            float* s_state, const int32_t* cu_seqlens, const int32_t* slots,
                                            const int64_t* positions, int entries, int num_heads, int dim, int vdim,
                                            int silu, int dtype, void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (entries < 0 || num_heads <= 0 || dim <= 0 || vdim <= 0 || proj_row_stride < (int64_t)num_heads * (2 * dim + vdim))
    return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || dim > 512 || num_heads > 65535 || vdim > 65535 * kCols) return MVLLM_ERR_UNSUPPORTED;
  if (entries == 0) return MVLLM_OK;
  if (!num || !proj || !decay || !s_state || !cu_seqlens || !slots || !positions) return MVLLM_ERR_NULL_POINTER;
  if (!aligned16(s_state)) return MVLLM_ERR_MISALIGNED;
  MemoryArgs a = {};
  a.num = num; a.proj = proj; a.s_state = s_state; a.cu = cu_seqlens; a.slot = slots; a.positions = positions;
  a.proj_stride = proj_row_stride; a.heads = num_heads; a.dim = dim; a.vdim = vdim; a.q_scale = 1.f; a.decay = decay;
  a.silu = silu;
  return dtype == MVLLM_F32 ? launch_recurrent<float, false>(a, entries, (hipStream_t)stream)
                            : launch_recurrent<bf16_t, false>(a, entries, (hipStream_t)stream);
}

extern "C" size_t mvllm_decay_memory_chunked_workspace_bytes(int num_segments, int num_heads, int dim, int vdim) {
  if (num_segments <= 0 || num_heads <= 0 || dim <= 0 || vdim <= 0) return 0;
  return (size_t)num_segments * num_heads * dim * vdim * sizeof(float);
}

extern "C" int mvllm_decay_memory_chunked(float* num, const void* proj, int64_t proj_row_stride, const float* log_decay,
                                          float* s_state, const int32_t* cu_seqlens, const int32_t* slots,
                                          const int64_t* positions, const int32_t* segments, int num_segments, int split,
                                          int num_heads, int dim, int vdim, int silu, int dtype, void* workspace,
                                          size_t workspace_bytes, void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (num_segments < 0 || num_heads <= 0 || dim <= 0 || vdim <= 0 || proj_row_stride < (int64_t)num_heads * (2 * dim + vdim))
    return MVLLM_ERR_BAD_SHAPE;
  if (dtype != MVLLM_BF16 || dim % 8 != 0 || vdim % 8 != 0 || proj_row_stride % 8 != 0 || dim > 256 || num_heads > 65535 ||
      proj_row_stride > (1 << 24) || vdim > (1 << 20) || (int64_t)num_heads * vdim > (1 << 22))
    return MVLLM_ERR_UNSUPPORTED;
  if (num_segments == 0) return MVLLM_OK;
  if (!num || !proj || !log_decay || !s_state || !cu_seqlens || !slots || !positions || !segments) return MVLLM_ERR_NULL_POINTER;
  if (!aligned16(proj)) return MVLLM_ERR_MISALIGNED;
  if (split && (!workspace || workspace_bytes < mvllm_decay_memory_chunked_workspace_bytes(num_segments, num_heads, dim, vdim)))
    return MVLLM_ERR_WORKSPACE;
  if (split && (!aligned16(workspace) || !aligned16(s_state))) return MVLLM_ERR_MISALIGNED;
  MemoryChunkArgs a = {};
  a.num = num; a.proj = reinterpret_cast<const bf16_t*>(proj); a.s_state = s_state; a.cu = cu_seqlens; a.slot = slots;
  a.positions = positions; a.segments = segments; a.ws_s = reinterpret_cast<float*>(workspace); a.proj_stride = proj_row_stride;
  a.num_segments = num_segments; a.heads = num_heads; a.dim = dim; a.vdim = vdim; a.q_scale = 1.f; a.log_decay = log_decay;
  a.silu = silu;
  return launch_chunked_sizes<false>(a, split != 0, (hipStream_t)stream);
}

extern "C" int mvllm_gated_row_norm(void* out, int64_t out_row_stride, const float* x, const float* weight, const void* gate,
                                    int64_t gate_row_stride, float eps, int64_t rows, int width, int dtype, void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || width <= 0 || gate_row_stride < width || out_row_stride < width) return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || rows > (1 << 30)) return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0) return MVLLM_OK;
  if (!out || !x || !weight || !gate) return MVLLM_ERR_NULL_POINTER;
  GatedNormArgs a;
  a.out = out; a.x = x; a.weight = weight; a.gate = gate; a.out_stride = out_row_stride; a.gate_stride = gate_row_stride;
  a.eps = eps; a.width = width;
  return dtype == MVLLM_F32 ? launch_gated_norm<float>(a, (int)rows, (hipStream_t)stream)
                            : launch_gated_norm<bf16_t>(a, (int)rows, (hipStream_t)stream);
}
