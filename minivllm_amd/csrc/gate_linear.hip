// Gate projections of a recurrent layer: out[T, N] = act(x[T, K] W[N, K]^T + bias), N small, fp32 accumulation and fp32
// output (a recurrence's gates enter exponentials, where a 16-bit result would be a few per cent off).  Columns below
// `split` get a soft cap, cap * tanh(z / cap), the others logsigmoid of the same.
//   bf16: one workgroup = 16 rows x 16 to 80 columns; its waves take 64-wide steps of K in turn on
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

constexpr int kFewRows = 512;        // up to here K is split over sixteen waves: the call is one memory round trip

// kWaves waves share K; NT column tiles per workgroup (one pass over x for all of them); kFull: K is a multiple of 64 and rows are 16-byte
// aligned, so that loads need no guards (rows and columns past the end load the last one and are not stored).
template <int kWaves, int NT, bool kFull>
__global__ __launch_bounds__(64 * kWaves) void gate_linear_bf16_kernel(const GateArgs a, bool vec) {
  __shared__ float4 part[kWaves][NT][64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int row = blockIdx.x * 16 + (lane & 15), col0 = blockIdx.y * 16 * NT + (lane & 15);
  const int k0 = 8 * (lane >> 4);
  const bf16_t* x = reinterpret_cast<const bf16_t*>(a.x) + (int64_t)(kFull ? min(row, a.rows - 1) : row) * a.x_stride;
  const bf16_t* w[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    const int col = col0 + 16 * n;
    w[n] = reinterpret_cast<const bf16_t*>(a.w) + (int64_t)(kFull ? min(col, a.N - 1) : col) * a.K;
  }
  v4f acc[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n) acc[n] = v4f{0.f, 0.f, 0.f, 0.f};
  if constexpr (kFull) {
#pragma unroll 4
    for (int k = 64 * wave + 2 * k0; k < a.K; k += 64 * kWaves) {      // a lane's 32 bytes: whole lines per row and wave
#pragma unroll
      for (int half = 0; half < 16; half += 8) {
        const uint4 xv = *reinterpret_cast<const uint4*>(x + k + half);
#pragma unroll
        for (int n = 0; n < NT; ++n) acc[n] = mfma16x16x32<bf16_t>(*reinterpret_cast<const uint4*>(w[n] + k + half), xv, acc[n]);
      }
    }
  } else {
#pragma unroll 4
    for (int k = 32 * wave; k < a.K; k += 32 * kWaves) {
      const uint4 xv = load_k8(x, k + k0, a.K, row < a.rows, vec);
#pragma unroll
      for (int n = 0; n < NT; ++n) acc[n] = mfma16x16x32<bf16_t>(load_k8(w[n], k + k0, a.K, col0 + 16 * n < a.N, vec), xv, acc[n]);
    }
  }
  // lane holds row l % 16, columns 4 (l / 16) + r of every tile; the activations are spread over the workgroup
#pragma unroll
  for (int n = 0; n < NT; ++n) part[wave][n][lane] = make_float4(acc[n][0], acc[n][1], acc[n][2], acc[n][3]);
  __syncthreads();
  for (int t = threadIdx.x; t < 256 * NT; t += 64 * kWaves) {
    const int n = t >> 8, c = (t >> 4) & 15, out_row = blockIdx.x * 16 + (t & 15), out_col = (blockIdx.y * NT + n) * 16 + c;
    if (out_row >= a.rows || out_col >= a.N) continue;
    float z = 0.f;
#pragma unroll
    for (int i = 0; i < kWaves; ++i) z += reinterpret_cast<const float*>(&part[i][n][16 * (c >> 2) + (t & 15)])[c & 3];
    a.out[(int64_t)out_row * a.N + out_col] = gate_activation(a, z, out_col);
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
  const unsigned tiles = (unsigned)((rows + 15) / 16);
  const dim3 grid(tiles, (unsigned)((N + 15) / 16));
  auto in_tiles = [&](int n) { return dim3(tiles, (unsigned)((N + 16 * n - 1) / (16 * n))); };
  hipStream_t s = (hipStream_t)stream;
  const bool vec = K % 8 == 0 && x_row_stride % 8 == 0 && aligned16(x) && aligned16(w), full = vec && K % 64 == 0;
  if (dtype == MVLLM_F32) gate_linear_f32_kernel<<<grid, dim3(256), 0, s>>>(a);
  else if (!full) gate_linear_bf16_kernel<4, 1, false><<<grid, dim3(256), 0, s>>>(a, vec);
  else if (rows <= kFewRows) gate_linear_bf16_kernel<16, 1, true><<<grid, dim3(1024), 0, s>>>(a, vec);
  else if (N <= 16) gate_linear_bf16_kernel<8, 1, true><<<grid, dim3(512), 0, s>>>(a, vec);
  else if (N <= 32) gate_linear_bf16_kernel<8, 2, true><<<in_tiles(2), dim3(512), 0, s>>>(a, vec);
  else if (N <= 48) gate_linear_bf16_kernel<8, 3, true><<<in_tiles(3), dim3(512), 0, s>>>(a, vec);
  else if (N <= 64) gate_linear_bf16_kernel<8, 4, true><<<in_tiles(4), dim3(512), 0, s>>>(a, vec);
  else gate_linear_bf16_kernel<8, 5, true><<<in_tiles(5), dim3(512), 0, s>>>(a, vec);
  return launch_status();
}
