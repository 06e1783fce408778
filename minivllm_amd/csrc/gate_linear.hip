// Gate projections of a recurrent layer: out[T, N] = act(x[T, K] W[N, K]^T + bias), N small, fp32 accumulation and fp32
// output (a recurrence's gates enter exponentials, where a 16-bit result would be a few per cent off).  Columns below
// `split` get a soft cap, cap * tanh(z / cap), the others logsigmoid of the same.
//   bf16: one workgroup = 16 rows x 16 columns; its four waves take 32-wide steps of K in turn on
//         v_mfma_f32_16x16x32_bf16 and meet in LDS.
//   fp32: the same tile with one fp32 dot product per thread over K chunks staged in LDS.
#include "common.h"

namespace mvllm {

struct GateArgs {
  float* out;              // [T, N]
  const void* x;           // [T, K]
  const void* w;           // [N, K]
  const float* bias;       // [N] or null
  int64_t x_stride;
  int rows, N, K, split;
  float cap;               // 0: no cap
};

__device__ __forceinline__ float gate_activation(const GateArgs& a, float z, int col) {
  if (a.bias) z += a.bias[col];
  if (a.cap > 0.f) z = a.cap * tanhf(z / a.cap);
  if (col >= a.split) z = fminf(z, 0.f) - log1pf(expf(-fabsf(z)));    // log sigmoid
  return z;
}

__device__ __forceinline__ uint4 load_k8(const bf16_t* row, int k, int K, bool live, bool vec) {
  uint4 r = make_uint4(0u, 0u, 0u, 0u);
  if (!live || k >= K) return r;
  if (vec && k + 8 <= K) return *reinterpret_cast<const uint4*>(row + k);
  bf16_t v[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) v[i].bits = k + i < K ? row[k + i].bits : (uint16_t)0;
  return *reinterpret_cast<const uint4*>(v);
}

__global__ __launch_bounds__(256) void gate_linear_bf16_kernel(const GateArgs a, bool vec) {
  __shared__ float4 part[3][64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int row = blockIdx.x * 16 + (lane & 15), col = blockIdx.y * 16 + (lane & 15);
  const bf16_t* x = reinterpret_cast<const bf16_t*>(a.x) + (int64_t)row * a.x_stride;
  const bf16_t* w = reinterpret_cast<const bf16_t*>(a.w) + (int64_t)col * a.K;
  const int k0 = 8 * (lane >> 4);
  v4f acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int k = 32 * wave; k < a.K; k += 128)
    acc = mfma16x16x32<bf16_t>(load_k8(w, k + k0, a.K, col < a.N, vec), load_k8(x, k + k0, a.K, row < a.rows, vec), acc);
  // lane holds row l % 16, columns 4 (l / 16) + r
  if (wave > 0) part[wave - 1][lane] = make_float4(acc[0], acc[1], acc[2], acc[3]);
  __syncthreads();
  if (wave > 0 || row >= a.rows) return;
#pragma unroll
  for (int i = 0; i < 3; ++i) {
    const float4 p = part[i][lane];
    acc[0] += p.x; acc[1] += p.y; acc[2] += p.z; acc[3] += p.w;
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int n = blockIdx.y * 16 + 4 * (lane >> 4) + r;
    if (n < a.N) a.out[(int64_t)row * a.N + n] = gate_activation(a, acc[r], n);
  }
}

__global__ __launch_bounds__(256) void gate_linear_f32_kernel(const GateArgs a) {
  constexpr int kStep = 64;
  __shared__ float xs[16][kStep + 1], ws[16][kStep + 1];
  const int r = threadIdx.x >> 4, c = threadIdx.x & 15;
  const int row = blockIdx.x * 16 + r, col = blockIdx.y * 16 + c;
  const float* x = reinterpret_cast<const float*>(a.x);
  const float* w = reinterpret_cast<const float*>(a.w);
  float acc = 0.f;
  for (int k0 = 0; k0 < a.K; k0 += kStep) {
    for (int i = threadIdx.x; i < 16 * kStep; i += 256) {
      const int rr = i / kStep, k = i % kStep;
      const int xr = blockIdx.x * 16 + rr, wr = blockIdx.y * 16 + rr;
      xs[rr][k] = xr < a.rows && k0 + k < a.K ? x[(int64_t)xr * a.x_stride + k0 + k] : 0.f;
      ws[rr][k] = wr < a.N && k0 + k < a.K ? w[(int64_t)wr * a.K + k0 + k] : 0.f;
    }
    __syncthreads();
#pragma unroll 16
    for (int k = 0; k < kStep; ++k) acc = fmaf(xs[r][k], ws[c][k], acc);
    __syncthreads();
  }
  if (row < a.rows && col < a.N) a.out[(int64_t)row * a.N + col] = gate_activation(a, acc, col);
}

}  // namespace mvllm

using namespace mvllm;

extern "C" int mvllm_gate_linear(float* out, const void* x, int64_t x_row_stride, const void* w, const float* bias,
                                 int64_t rows, int N, int K, int split, float cap, int dtype, void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || N <= 0 || K <= 0 || split < 0 || split > N || x_row_stride < K || !(cap >= 0.f)) return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || rows > (1 << 30) || N > 65535 * 16) return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0) return MVLLM_OK;
  if (!out || !x || !w) return MVLLM_ERR_NULL_POINTER;
  GateArgs a;
  a.out = out; a.x = x; a.w = w; a.bias = bias; a.x_stride = x_row_stride; a.rows = (int)rows; a.N = N; a.K = K;
  a.split = split; a.cap = cap;
  const dim3 grid((unsigned)((rows + 15) / 16), (unsigned)((N + 15) / 16));
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MVLLM_F32) gate_linear_f32_kernel<<<grid, dim3(256), 0, s>>>(a);
  else gate_linear_bf16_kernel<<<grid, dim3(256), 0, s>>>(a, K % 8 == 0 && x_row_stride % 8 == 0 && aligned16(x) && aligned16(w));
  return launch_status();
}
