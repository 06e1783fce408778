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
// Recurrence kernel: one workgroup = (entry, head, 64 value columns).  A thread holds 4 columns of every 16th row of S
// in registers (kRows of them), sixteen threads side by side cover the columns and sixteen such groups the rows.
#include "common.h"

#pragma clang fp contract(off)

namespace mvllm {

constexpr int kCols = 64;            // value columns per workgroup

struct MlstmArgs {
  float* num;                // [T, H, vdim]
  float* den;                // [T, H]
  float* m_next;             // [entries, H]: running maximum after the entry's last row
  const void* proj;          // [T, proj_stride]: q at 0, k at H dim, v at 2 H dim
  const float* gates;        // [T, 2 H]: log input gates, log forget gates
  float* s_state;            // [slots, H, dim, vdim]
  float* n_state;            // [slots, H, dim]
  const float* m_state;      // [slots, H]
  const int32_t* cu;         // [entries + 1] rows
  const int32_t* slot;       // [entries]
  const int64_t* positions;  // [T]
  int64_t proj_stride;
  int heads, dim, vdim;
  float q_scale, floor;
};

template <typename T, int kRows>
__global__ __launch_bounds__(256) void mlstm_recurrent_kernel(const MlstmArgs a) {
  __shared__ float qs[16 * kRows], ks[16 * kRows], part[4][kCols], red[4];
  const int entry = blockIdx.x, h = blockIdx.y, tile = blockIdx.z;
  const int row0 = a.cu[entry], row1 = a.cu[entry + 1];
  const int slot = a.slot[entry];
  if (row0 >= row1 || slot < 0) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int dim = a.dim, vdim = a.vdim;
  const int col0 = tile * kCols + 4 * (tid & 15), rg = tid >> 4;
  const int ncols = min(4, vdim - col0);                 // may be <= 0
  const bool vec = vdim % 4 == 0 && ncols == 4;
  const bool fresh = a.positions[row0] == 0;
  float* s_ptr = a.s_state + ((int64_t)slot * a.heads + h) * dim * vdim;
  float* n_ptr = a.n_state + ((int64_t)slot * a.heads + h) * dim;
  float m = fresh ? 0.f : a.m_state[(int64_t)slot * a.heads + h];
  float s[kRows][4];
#pragma unroll
  for (int r = 0; r < kRows; ++r) {
    const int d = rg + 16 * r;
#pragma unroll
    for (int c = 0; c < 4; ++c) s[r][c] = 0.f;
    if (!fresh && d < dim && ncols > 0) {
      const float* p = s_ptr + (int64_t)d * vdim + col0;
      if (vec) {
        const float4 f = *reinterpret_cast<const float4*>(p);
        s[r][0] = f.x; s[r][1] = f.y; s[r][2] = f.z; s[r][3] = f.w;
      } else {
#pragma unroll
        for (int c = 0; c < 4; ++c)
          if (c < ncols) s[r][c] = p[c];
      }
    }
  }
  // tile 0 also carries n, one or two dims per thread
  constexpr int kN = (16 * kRows + 255) / 256;
  float n[kN];
  if (tile == 0) {
#pragma unroll
    for (int i = 0; i < kN; ++i) {
      const int d = tid + 256 * i;
      n[i] = !fresh && d < dim ? n_ptr[d] : 0.f;
    }
  }
  const T* base = reinterpret_cast<const T*>(a.proj);
  for (int row = row0; row < row1; ++row) {
    const T* p = base + (int64_t)row * a.proj_stride;
    for (int d = tid; d < 16 * kRows; d += 256) {
      qs[d] = d < dim ? to_float(p[(int64_t)h * dim + d]) * a.q_scale : 0.f;
      ks[d] = d < dim ? to_float(p[(int64_t)(a.heads + h) * dim + d]) : 0.f;
    }
    const float gi = a.gates[(int64_t)row * 2 * a.heads + h], gf = a.gates[(int64_t)row * 2 * a.heads + a.heads + h];
    const float m_new = fmaxf(gf + m, gi);
    const float keep = expf(gf + m - m_new), add = expf(gi - m_new);
    m = m_new;
    float v[4];
#pragma unroll
    for (int c = 0; c < 4; ++c) v[c] = c < ncols ? to_float(p[(int64_t)2 * a.heads * dim + (int64_t)h * vdim + col0 + c]) * add : 0.f;
    __syncthreads();
    float acc[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int r = 0; r < kRows; ++r) {
      const float kd = ks[rg + 16 * r], qd = qs[rg + 16 * r];
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        s[r][c] = fmaf(kd, v[c], keep * s[r][c]);
        acc[c] = fmaf(s[r][c], qd, acc[c]);
      }
    }
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      acc[c] += __shfl_xor(acc[c], 16, 64);
      acc[c] += __shfl_xor(acc[c], 32, 64);
    }
    if (lane < 16) {
#pragma unroll
      for (int c = 0; c < 4; ++c) part[wave][4 * lane + c] = acc[c];
    }
    if (tile == 0) {
      float dot = 0.f;
#pragma unroll
      for (int i = 0; i < kN; ++i) {
        const int d = tid + 256 * i;
        if (d < 16 * kRows) {
          n[i] = fmaf(add, ks[d], keep * n[i]);
          dot = fmaf(n[i], qs[d], dot);
        }
      }
      dot = wave_sum(dot);
      if (lane == 0) red[wave] = dot;
    }
    __syncthreads();
    if (tid < kCols && tile * kCols + tid < vdim)
      a.num[((int64_t)row * a.heads + h) * vdim + tile * kCols + tid] = part[0][tid] + part[1][tid] + part[2][tid] + part[3][tid];
    if (tile == 0 && tid == 0)
      a.den[(int64_t)row * a.heads + h] = fmaxf(fabsf(red[0] + red[1] + red[2] + red[3]), expf(-m)) + a.floor;
    // qs, ks and part are written again only after this row's readers have passed the next row's first barrier or, for
    // qs and ks, this one: they were last read before it
  }
#pragma unroll
  for (int r = 0; r < kRows; ++r) {
    const int d = rg + 16 * r;
    if (d < dim && ncols > 0) {
      float* p = s_ptr + (int64_t)d * vdim + col0;
      if (vec) *reinterpret_cast<float4*>(p) = make_float4(s[r][0], s[r][1], s[r][2], s[r][3]);
      else {
#pragma unroll
        for (int c = 0; c < 4; ++c)
          if (c < ncols) p[c] = s[r][c];
      }
    }
  }
  if (tile == 0) {
#pragma unroll
    for (int i = 0; i < kN; ++i) {
      const int d = tid + 256 * i;
      if (d < dim) n_ptr[d] = n[i];
    }
    if (tid == 0) a.m_next[(int64_t)entry * a.heads + h] = m;
  }
}

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

template <typename T>
static int launch_recurrent(const MlstmArgs& a, int entries, hipStream_t stream) {
  const dim3 grid((unsigned)entries, (unsigned)a.heads, (unsigned)((a.vdim + kCols - 1) / kCols)), block(256);
  if (a.dim <= 64) mlstm_recurrent_kernel<T, 4><<<grid, block, 0, stream>>>(a);
  else if (a.dim <= 128) mlstm_recurrent_kernel<T, 8><<<grid, block, 0, stream>>>(a);
  else if (a.dim <= 256) mlstm_recurrent_kernel<T, 16><<<grid, block, 0, stream>>>(a);
  else mlstm_recurrent_kernel<T, 32><<<grid, block, 0, stream>>>(a);
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
  MlstmArgs a;
  a.num = num; a.den = den; a.m_next = m_next; a.proj = proj; a.gates = gates; a.s_state = s_state; a.n_state = n_state;
  a.m_state = m_state; a.cu = cu_seqlens; a.slot = slots; a.positions = positions; a.proj_stride = proj_row_stride;
  a.heads = num_heads; a.dim = dim; a.vdim = vdim; a.q_scale = q_scale; a.floor = floor;
  return dtype == MVLLM_F32 ? launch_recurrent<float>(a, entries, (hipStream_t)stream)
                            : launch_recurrent<bf16_t>(a, entries, (hipStream_t)stream);
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
