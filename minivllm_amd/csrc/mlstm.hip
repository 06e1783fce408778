// The matrix-memory recurrence of the mLSTM (exponential gates, running maximum), token by token, and what follows it.
//     m' = max(f + m, i);  keep = exp(f + m - m'), add = exp(i - m')
//     S  = keep S + add k v^T;  n = keep n + add k                       (S [dim, vdim], n [dim], fp32)
//     num = S^T q;  den = max(|n . q|, exp(-m')) + floor
// mvllm_mlstm_recurrent runs every row of every entry through it: the decode form (one row per entry: S is read and
// written once) and the exact form for short portions and for fp32.
// mvllm_mlstm_output: out = rms(num / den) per head * weight * sigmoid(gate), and the new running maximum into the state
// (every workgroup of a head reads the old one, so nobody writes it while they run).
// State of a slot: S [H, dim, vdim], n [H, dim], m [H], all fp32; an entry whose first row is at position 0 starts from
// zeros whatever the slot holds.
//
// The recurrence kernel is memory_recurrent.h's.
#include "memory_recurrent.h"

#pragma clang fp contract(off)

namespace mvllm {

struct MlstmOutArgs {
  void* out;                 // [T, H * vdim]
  const float* num;          // [T, H, vdim]
  const float* den;          // [T, H]
  const float* weight;       // [H * vdim]
  const void* gate;          // [T, gate_stride]: H * vdim pre-activations per row
  const float* m_next;       // [entries, H]
  float* m_state;            // [slots, H]
  const int32_t* cu;
  const int32_t* row_entry;
  const int32_t* slot;
  int64_t gate_stride;
  int64_t rows;
  int heads, vdim;
  float eps;
};

// The new running maximum of a (row, head) into the state, if the row is its entry's last one.
template <typename A> __device__ __forceinline__ void keep_max(const A& a, int64_t row, int h) {
  const int entry = a.row_entry[row];
  if (row + 1 == a.cu[entry + 1] && a.slot[entry] >= 0)
    a.m_state[(int64_t)a.slot[entry] * a.heads + h] = a.m_next[(int64_t)entry * a.heads + h];
}

// kItems consecutive (row, head) per wave, four columns per lane: vdim a multiple of 4 and at most 256.
template <typename T, int kItems>
__global__ __launch_bounds__(256) void mlstm_output_kernel(const MlstmOutArgs a) {
  const int lane = threadIdx.x & 63, c = 4 * lane;
  const uint32_t item0 = (blockIdx.x * 4 + (threadIdx.x >> 6)) * kItems, items = (uint32_t)a.rows * (uint32_t)a.heads;
  if (item0 >= items) return;
  const uint32_t row0 = item0 / (uint32_t)a.heads, h0 = item0 - row0 * (uint32_t)a.heads;
  float4 num[kItems], w[kItems];
  float g[kItems][4], inv_den[kItems];
  const float inv_vdim = 1.0f / (float)a.vdim;
  const bool has = c < a.vdim;
  uint32_t row = row0, h = h0;
#pragma unroll
  for (int i = 0; i < kItems; ++i) {
    num[i] = w[i] = make_float4(0.f, 0.f, 0.f, 0.f);
    g[i][0] = g[i][1] = g[i][2] = g[i][3] = 0.f;
    inv_den[i] = 0.f;
    if (item0 + i < items) {
      inv_den[i] = __builtin_amdgcn_rcpf(a.den[item0 + i]);
      if (has) {
        const T* gate = reinterpret_cast<const T*>(a.gate) + row * a.gate_stride + (int64_t)h * a.vdim + c;
        num[i] = *reinterpret_cast<const float4*>(a.num + (int64_t)(item0 + i) * a.vdim + c);
        w[i] = *reinterpret_cast<const float4*>(a.weight + (int64_t)h * a.vdim + c);
        if constexpr (sizeof(T) == 4) {
          const float4 gv = *reinterpret_cast<const float4*>(gate);
          g[i][0] = gv.x; g[i][1] = gv.y; g[i][2] = gv.z; g[i][3] = gv.w;
        } else {
          const uint2 gv = *reinterpret_cast<const uint2*>(gate);
          g[i][0] = lo_to_float<T>(gv.x); g[i][1] = hi_to_float<T>(gv.x); g[i][2] = lo_to_float<T>(gv.y); g[i][3] = hi_to_float<T>(gv.y);
        }
      }
    }
    if (++h == (uint32_t)a.heads) { h = 0; ++row; }
  }
  row = row0;
  h = h0;
#pragma unroll
  for (int i = 0; i < kItems; ++i) {
    if (item0 + i >= items) return;
    const float x[4] = {num[i].x * inv_den[i], num[i].y * inv_den[i], num[i].z * inv_den[i], num[i].w * inv_den[i]};
    const float ss = four_rows_sum(row16_sum(x[0] * x[0] + x[1] * x[1] + x[2] * x[2] + x[3] * x[3]));
    const float s = __builtin_amdgcn_rsqf(ss * inv_vdim + a.eps);
    const float wv[4] = {w[i].x, w[i].y, w[i].z, w[i].w};
    if (has) {
      T r[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) r[e] = from_float<T>(x[e] * s * wv[e] * __builtin_amdgcn_rcpf(1.0f + __expf(-g[i][e])));
      T* out = reinterpret_cast<T*>(a.out) + (int64_t)(item0 + i) * a.vdim + c;
      if constexpr (sizeof(T) == 4) store16_stream(out, *reinterpret_cast<const uint4*>(r));
      else store8_stream(out, *reinterpret_cast<const uint2*>(r));
    }
    if (lane == 0) keep_max(a, row, (int)h);
    if (++h == (uint32_t)a.heads) { h = 0; ++row; }
  }
}

// One (row, head) per wave, any vdim.
template <typename T>
__global__ __launch_bounds__(256) void mlstm_output_any_kernel(const MlstmOutArgs a) {
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  if (item >= a.rows * a.heads) return;
  const int64_t row = item / a.heads;
  const int h = (int)(item - row * a.heads);
  const float* num = a.num + item * a.vdim;
  const T* gate = reinterpret_cast<const T*>(a.gate) + row * a.gate_stride + (int64_t)h * a.vdim;
  const float* weight = a.weight + (int64_t)h * a.vdim;
  T* out = reinterpret_cast<T*>(a.out) + item * a.vdim;
  const float inv_den = 1.0f / a.den[item];
  float ss = 0.f;
  for (int c = lane; c < a.vdim; c += 64) {
    const float x = num[c] * inv_den;
    ss = fmaf(x, x, ss);
  }
  const float s = 1.0f / sqrtf(wave_sum(ss) / (float)a.vdim + a.eps) * inv_den;
  for (int c = lane; c < a.vdim; c += 64)
    out[c] = from_float<T>(num[c] * s * weight[c] / (1.0f + __expf(-to_float(gate[c]))));
  if (lane == 0) keep_max(a, row, h);
}

template <typename T>
static int launch_output(const MlstmOutArgs& a, bool vec, hipStream_t stream) {
  const int64_t items = a.rows * a.heads;
  if (!vec) mlstm_output_any_kernel<T><<<dim3((unsigned)((items + 3) / 4)), dim3(256), 0, stream>>>(a);
  else if (items < 16384) mlstm_output_kernel<T, 1><<<dim3((unsigned)((items + 3) / 4)), dim3(256), 0, stream>>>(a);
  else mlstm_output_kernel<T, 4><<<dim3((unsigned)((items + 15) / 16)), dim3(256), 0, stream>>>(a);
  return launch_status();
}

}  // namespace mvllm

using namespace mvllm;

extern "C" int mvllm_mlstm_recurrent(float* num, float* den, float* m_next, const void* proj, int64_t proj_row_stride,
                                     const float* gates, float* s_state, float* n_state, const float* m_state,
                                     const int32_t* cu_seqlens, const int32_t* slots, const int64_t* positions, int entries,
                                     int num_heads, int dim, int vdim, float q_scale, float floor, int dtype, void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (entries < 0 || num_heads <= 0 || dim <= 0 || vdim <= 0 || proj_row_stride < (int64_t)num_heads * (2 * dim + vdim))
    return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || dim > 512 || num_heads > 65535 || vdim > 65535 * kCols) return MVLLM_ERR_UNSUPPORTED;
  if (entries == 0) return MVLLM_OK;
  if (!num || !den || !m_next || !proj || !gates || !s_state || !n_state || !m_state || !cu_seqlens || !slots || !positions)
    return MVLLM_ERR_NULL_POINTER;
  if (!aligned16(s_state)) return MVLLM_ERR_MISALIGNED;
  MemoryArgs a = {};
  a.num = num; a.den = den; a.m_next = m_next; a.proj = proj; a.gates = gates; a.s_state = s_state; a.n_state = n_state;
  a.m_state = m_state; a.cu = cu_seqlens; a.slot = slots; a.positions = positions; a.proj_stride = proj_row_stride;
  a.heads = num_heads; a.dim = dim; a.vdim = vdim; a.q_scale = q_scale; a.floor = floor;
  return dtype == MVLLM_F32 ? launch_recurrent<float, true>(a, entries, (hipStream_t)stream)
                            : launch_recurrent<bf16_t, true>(a, entries, (hipStream_t)stream);
}

extern "C" int mvllm_mlstm_output(void* out, const float* num, const float* den, const float* weight, const void* gate,
                                  int64_t gate_row_stride, float eps, const float* m_next, float* m_state,
                                  const int32_t* cu_seqlens, const int32_t* row_entry, const int32_t* slots, int64_t rows,
                                  int num_heads, int vdim, int dtype, void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || num_heads <= 0 || vdim <= 0 || gate_row_stride < (int64_t)num_heads * vdim) return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || rows > ((int64_t)1 << 31) / num_heads) return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0) return MVLLM_OK;
  if (!out || !num || !den || !weight || !gate || !m_next || !m_state || !cu_seqlens || !row_entry || !slots) return MVLLM_ERR_NULL_POINTER;
  const uintptr_t gate_align = dtype == MVLLM_F32 ? 15u : 7u;
  const bool vec = vdim % 4 == 0 && vdim <= 256 && gate_row_stride % 4 == 0 && aligned16(num) && aligned16(out) && aligned16(weight) &&
                   (reinterpret_cast<uintptr_t>(gate) & gate_align) == 0;
  MlstmOutArgs a;
  a.out = out; a.num = num; a.den = den; a.weight = weight; a.gate = gate; a.m_next = m_next; a.m_state = m_state;
  a.cu = cu_seqlens; a.row_entry = row_entry; a.slot = slots; a.gate_stride = gate_row_stride; a.rows = rows;
  a.heads = num_heads; a.vdim = vdim; a.eps = eps;
  return dtype == MVLLM_F32 ? launch_output<float>(a, vec, (hipStream_t)stream) : launch_output<bf16_t>(a, vec, (hipStream_t)stream);
}
