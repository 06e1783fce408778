// Matrix memory, row by row: every row of an entry updates S [dim, vdim] and reads it.
//   gates:     the mLSTM's exponential gates with a running maximum and a normaliser (mlstm.hip has the equations)
//   no gates:  S = decay S + k v^T, num = S^T q, decay a constant of the head (decay_memory.hip)
// State of a slot: S [H, dim, vdim] (with gates also n [H, dim], m [H]), all fp32; an entry whose first row is at position
// 0 starts from zeros whatever the slot holds.
//
// One workgroup = (entry, head, 64 value columns).  A thread holds 4 columns of every 16th row of S in registers (kRows of
// them), sixteen threads side by side cover the columns and sixteen such groups the rows.
#pragma once
#include "common.h"

#pragma clang fp contract(off)

namespace mvllm {

constexpr int kCols = 64;            // value columns per workgroup

struct MemoryArgs {
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
  const float* decay;        // [H], without gates
  int silu;                  // q, k and v are taken through z * sigmoid(z)
};

__device__ __forceinline__ float silu(float z) { return z / (1.0f + __expf(-z)); }

template <typename T, int kRows, bool kGates>
__global__ __launch_bounds__(256) void memory_recurrent_kernel(const MemoryArgs a) {
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
  float* n_ptr = !kGates ? nullptr : a.n_state + ((int64_t)slot * a.heads + h) * dim;
  float m = 0.f, keep = 1.f, add = 1.f;
  if constexpr (kGates) m = fresh ? 0.f : a.m_state[(int64_t)slot * a.heads + h];
  else keep = a.decay[h];
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
  if (kGates && tile == 0) {
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
      float q = d < dim ? to_float(p[(int64_t)h * dim + d]) : 0.f, k = d < dim ? to_float(p[(int64_t)(a.heads + h) * dim + d]) : 0.f;
      if (!kGates && a.silu) {
        q = silu(q);
        k = silu(k);
      }
      qs[d] = q * a.q_scale;
      ks[d] = k;
    }
    if constexpr (kGates) {
      const float gi = a.gates[(int64_t)row * 2 * a.heads + h], gf = a.gates[(int64_t)row * 2 * a.heads + a.heads + h];
      const float m_new = fmaxf(gf + m, gi);
      keep = expf(gf + m - m_new);
      add = expf(gi - m_new);
      m = m_new;
    }
    float v[4];
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      v[c] = c < ncols ? to_float(p[(int64_t)2 * a.heads * dim + (int64_t)h * vdim + col0 + c]) : 0.f;
      if (!kGates && a.silu) v[c] = silu(v[c]);
      v[c] *= add;
    }
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
    if (kGates && tile == 0) {
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
    if (kGates && tile == 0 && tid == 0)
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
  if (kGates && tile == 0) {
#pragma unroll
    for (int i = 0; i < kN; ++i) {
      const int d = tid + 256 * i;
      if (d < dim) n_ptr[d] = n[i];
    }
    if (tid == 0) a.m_next[(int64_t)entry * a.heads + h] = m;
  }
}

template <typename T, bool kGates>
static int launch_recurrent(const MemoryArgs& a, int entries, hipStream_t stream) {
  const dim3 grid((unsigned)entries, (unsigned)a.heads, (unsigned)((a.vdim + kCols - 1) / kCols)), block(256);
  if (a.dim <= 64) memory_recurrent_kernel<T, 4, kGates><<<grid, block, 0, stream>>>(a);
  else if (a.dim <= 128) memory_recurrent_kernel<T, 8, kGates><<<grid, block, 0, stream>>>(a);
  else if (a.dim <= 256) memory_recurrent_kernel<T, 16, kGates><<<grid, block, 0, stream>>>(a);
  else memory_recurrent_kernel<T, 32, kGates><<<grid, block, 0, stream>>>(a);
  return launch_status();
}

}  // namespace mvllm
