// Rows spread over a workgroup: loads and stores of a thread's channels, and sums over the workgroup.
#pragma once
#include "common.h"

#pragma clang fp contract(off)

namespace mvllm {

constexpr int kMaxThreads = 1024;

template <typename T, int VEC> struct Chunk;
template <> struct Chunk<float, 4> {
  static __device__ __forceinline__ void load(const float* p, float* v) {
    const float4 f = *reinterpret_cast<const float4*>(p);
    v[0] = f.x; v[1] = f.y; v[2] = f.z; v[3] = f.w;
  }
  static __device__ __forceinline__ void store(float* p, const float* v) {
    store16_stream(p, make_uint4(__float_as_uint(v[0]), __float_as_uint(v[1]), __float_as_uint(v[2]), __float_as_uint(v[3])));
  }
};
template <> struct Chunk<bf16_t, 4> {
  static __device__ __forceinline__ void load(const bf16_t* p, float* v) {
    const uint2 w = *reinterpret_cast<const uint2*>(p);
    v[0] = lo_to_float<bf16_t>(w.x); v[1] = hi_to_float<bf16_t>(w.x);
    v[2] = lo_to_float<bf16_t>(w.y); v[3] = hi_to_float<bf16_t>(w.y);
  }
  static __device__ __forceinline__ void store(bf16_t* p, const float* v) {
    bf16_t r[4];
    for (int i = 0; i < 4; ++i) r[i] = from_float<bf16_t>(v[i]);
    store8_stream(p, *reinterpret_cast<const uint2*>(r));
  }
};
template <typename T> struct Chunk<T, 1> {
  static __device__ __forceinline__ void load(const T* p, float* v) { v[0] = to_float(*p); }
  static __device__ __forceinline__ void store(T* p, const float* v) { *p = from_float<T>(v[0]); }
};

// Sums of N values per thread over the workgroup, the same in every thread: rows of 16 lanes in registers, the rows of all
// waves (at most 64) through LDS.  Consecutive calls take the two halves of `lds` in turn (`flip`): whoever writes a half
// again has passed the barrier of the call in between, which everybody reaches after reading it.
template <int N>
__device__ __forceinline__ void block_sums(float* v, float* lds, int waves, int& flip) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
#pragma unroll
  for (int i = 0; i < N; ++i) v[i] = row16_sum(v[i]);
  if (waves > 1) {
    lds += flip * (kMaxThreads / 16) * N;
    flip ^= 1;
    if ((lane & 15) == 0) {
#pragma unroll
      for (int i = 0; i < N; ++i) lds[(wave * 4 + (lane >> 4)) * N + i] = v[i];
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] = row16_sum(lane < 4 * waves ? lds[lane * N + i] : 0.f);
  }
#pragma unroll
  for (int i = 0; i < N; ++i) v[i] = four_rows_sum(v[i]);
}

}  // namespace mvllm
