// Attention over latents: the cache keeps one row c [rank] per token, and per head k = U_k c, v = U_v c.  Since
//     q . (U_k c) = (U_k^T q) . c        and        sum_j p_j U_v c_j = U_v (sum_j p_j c_j)
// a query row can be answered from the latents alone: q' = U_k^T q per head (head_linear), softmax over q' . c with the
// latents as both keys and values (latent_decode: all heads of a row read a latent once), then U_v per head (head_linear).
// That is the form for decoded tokens and short portions; long portions make keys and values of the latents (a matrix
// product) and run the prefill kernels.
//   latent_norm_store   c = rms(row) * weight, packed and into the cache
//   latent_rope_store   the same with a rotated part behind the latent, and another norm (the queries' latent) beside it
//   head_linear         out[t, h] = W_h x[t, h]
//   latent_decode       one query row per (row, block of heads, share of the keys); latent_merge joins the shares
// The rank is padded to a multiple of 32 with zeros; scores, weights and sums are fp32.
#include "latent_decode.h"

#pragma clang fp contract(off)

namespace mvllm {

// ---- norm and store ----
struct LatentNormArgs {
  void* out;                // [*, padded] or null
  const int64_t* out_rows;  // [T]: row of `out` (< 0: none), or null: row t
  const void* in;           // [T, in_stride]
  const float* weight;      // [rank]
  void* cache;              // [num_slots, padded] or null
  const int64_t* slots;     // [T], < 0: not stored
  const float2* rot_table;  // [max_position, rot_dims / 2] (cos, sin) or null
  const int64_t* positions; // [T]
  int64_t in_stride, num_slots, max_position;
  float eps;
  int rows, rank, padded;
  int rot_col, rot, rot_dims, interleaved;   // columns rot_col .. rot_col + rot are not normed; their first rot_dims turn
  bool vec;                 // the weight starts on 16 bytes
};

// Column `d` of the rotated part of a row, its partner read from memory; pairs (2i, 2i + 1) or (i, i + dims / 2).
template <typename T>
__device__ __forceinline__ float turned_column(const LatentNormArgs& a, const T* part, const float2* cs, float own, int d) {
  if (d >= a.rot_dims) return own;
  const int half = a.rot_dims / 2;
  const bool low = a.interleaved ? (d & 1) == 0 : d < half;
  const int pair = a.interleaved ? d >> 1 : low ? d : d - half, other = a.interleaved ? d ^ 1 : low ? d + half : d - half;
  const float2 c = cs[pair];
  const float p = to_float(part[other]);
  return low ? own * c.x - p * c.y : own * c.x + p * c.y;
}

// One row per wave, 16 bytes per lane and access; blockIdx.y: which of two norms.
template <typename T, int NC>
__global__ __launch_bounds__(256) void latent_norm_kernel(const LatentNormArgs first, const LatentNormArgs second) {
  constexpr int N = 16 / (int)sizeof(T);
  const LatentNormArgs& a = blockIdx.y == 0 ? first : second;
  const int row = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (row >= a.rows) return;
  const T* in = reinterpret_cast<const T*>(a.in) + (int64_t)row * a.in_stride;
  const int64_t slot = a.slots ? a.slots[row] : -1;
  const int64_t out_row = a.out_rows ? a.out_rows[row] : row;
  const bool turns = a.rot_table != nullptr;
  const int64_t pos = turns ? a.positions[row] : 0;
  float x[NC][N], w[NC][N], ss = 0.f;
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int at = (c * 64 + lane) * N;
    if (at + N <= a.rank && a.vec) {
#pragma unroll
      for (int i = 0; i < N; i += 4) *reinterpret_cast<float4*>(&w[c][i]) = *reinterpret_cast<const float4*>(a.weight + at + i);
    } else if (at < a.rank) {
#pragma unroll
      for (int i = 0; i < N; ++i) w[c][i] = a.weight[min(at + i, a.rank - 1)];
    }
  }
  const float2* cs = turns ? a.rot_table + min(max(pos, (int64_t)0), a.max_position - 1) * (a.rot_dims / 2) : nullptr;
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int at = (c * 64 + lane) * N;
    T v[N];
    if (at < a.padded) *reinterpret_cast<uint4*>(v) = *reinterpret_cast<const uint4*>(in + at);
#pragma unroll
    for (int i = 0; i < N; ++i) {
      x[c][i] = at + i < a.rank ? to_float(v[i]) : 0.f;
      ss = fmaf(x[c][i], x[c][i], ss);
    }
    if (turns && at + N > a.rot_col && at < a.rot_col + a.rot) {         // (the parts start on multiples of N: all or none)
#pragma unroll
      for (int i = 0; i < N; ++i)
        if (at + i < a.rot_col + a.rot) x[c][i] = turned_column(a, in + a.rot_col, cs, to_float(v[i]), at + i - a.rot_col);
    }
  }
  ss = four_rows_sum(row16_sum(ss));
  const float inv = 1.0f / sqrtf(ss / (float)a.rank + a.eps);
  T* out = a.out && out_row >= 0 ? reinterpret_cast<T*>(a.out) + out_row * a.padded : nullptr;
  T* cached = a.cache && slot >= 0 && slot < a.num_slots ? reinterpret_cast<T*>(a.cache) + slot * a.padded : nullptr;
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int at = (c * 64 + lane) * N;
    if (at >= a.padded) continue;
    T v[N];
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] = from_float<T>(at + i < a.rank ? x[c][i] * inv * w[c][i] : x[c][i]);
    const uint4 r = *reinterpret_cast<const uint4*>(v);
    if (out) *reinterpret_cast<uint4*>(out + at) = r;
    if (cached) *reinterpret_cast<uint4*>(cached + at) = r;
  }
}

template <typename T>
static void launch_latent_norm(const LatentNormArgs& a, const LatentNormArgs& b, bool two, hipStream_t s) {
  const dim3 grid((unsigned)((a.rows + 3) / 4), two ? 2 : 1), block(256);
  const int widest = two && b.padded > a.padded ? b.padded : a.padded;
  constexpr int kFew = sizeof(T) == 4 ? 2 : 1;
  if (widest <= 512) latent_norm_kernel<T, kFew><<<grid, block, 0, s>>>(a, b);
  else if (widest <= 1024) latent_norm_kernel<T, 2 * kFew><<<grid, block, 0, s>>>(a, b);
  else latent_norm_kernel<T, 4 * kFew><<<grid, block, 0, s>>>(a, b);
}

// ---- a matrix per head ----
struct HeadLinearArgs {
  void* out;                // [rows, H, N] with strides
  const void* x;            // [rows, H, K] with strides
  const void* w;            // [H, N, K] dense
  int64_t out_row, out_head, x_row, x_head;
  int rows, heads, N, K;
};

// Workgroup = 16 RT rows, one head.  kSplitK: 16 outputs, the waves share K and meet in LDS; otherwise 64 outputs, 16 per
// wave.  K a multiple of 8, N of 16.  Rows and K past the end read the last ones; what they would add is multiplied by zeros
// or not stored.
template <int RT, bool kSplitK>
__global__ __launch_bounds__(256) void head_linear_bf16_kernel(const HeadLinearArgs a) {
  __shared__ float4 part[kSplitK ? 4 : 1][kSplitK ? RT : 1][kSplitK ? 64 : 1];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, g = lane >> 4, i16 = lane & 15;
  const int h = blockIdx.y, n0 = kSplitK ? blockIdx.x * 16 : (blockIdx.x * 4 + wave) * 16;
  if (!kSplitK && n0 >= a.N) return;
  const int row0 = blockIdx.z * 16 * RT + i16;
  const bf16_t* x[RT];
#pragma unroll
  for (int t = 0; t < RT; ++t)
    x[t] = reinterpret_cast<const bf16_t*>(a.x) + (int64_t)min(row0 + 16 * t, a.rows - 1) * a.x_row + (int64_t)h * a.x_head;
  const bf16_t* w = reinterpret_cast<const bf16_t*>(a.w) + ((int64_t)h * a.N + n0 + i16) * a.K;
  v4f acc[RT];
#pragma unroll
  for (int t = 0; t < RT; ++t) acc[t] = v4f{0.f, 0.f, 0.f, 0.f};
  const uint4 zero = make_uint4(0u, 0u, 0u, 0u);
#pragma unroll 4
  for (int k0 = kSplitK ? 32 * wave : 0; k0 < a.K; k0 += kSplitK ? 128 : 32) {
    const int k = min(k0 + 8 * g, a.K - 8);
    uint4 wv = *reinterpret_cast<const uint4*>(w + k), xv[RT];
#pragma unroll
    for (int t = 0; t < RT; ++t) xv[t] = *reinterpret_cast<const uint4*>(x[t] + k);
    if (k0 + 8 * g >= a.K) {
      wv = zero;
#pragma unroll
      for (int t = 0; t < RT; ++t) xv[t] = zero;
    }
#pragma unroll
    for (int t = 0; t < RT; ++t) acc[t] = mfma16x16x32<bf16_t>(wv, xv[t], acc[t]);
  }
  // lane: row i16 of a tile, outputs n0 + 4 g + r
  auto store = [&](int t, float4 o) __attribute__((always_inline)) {
    const int row = row0 + 16 * t;
    if (row >= a.rows) return;
    bf16_t* out = reinterpret_cast<bf16_t*>(a.out) + (int64_t)row * a.out_row + (int64_t)h * a.out_head + n0 + 4 * g;
    *reinterpret_cast<uint2*>(out) = make_uint2(pack2<bf16_t>(o.x, o.y), pack2<bf16_t>(o.z, o.w));
  };
  if constexpr (!kSplitK) {
#pragma unroll
    for (int t = 0; t < RT; ++t) store(t, make_float4(acc[t][0], acc[t][1], acc[t][2], acc[t][3]));
  } else {
#pragma unroll
    for (int t = 0; t < RT; ++t) part[wave][t][lane] = make_float4(acc[t][0], acc[t][1], acc[t][2], acc[t][3]);
    __syncthreads();
    for (int t = wave; t < RT; t += 4) {
      float4 o = part[0][t][lane];
#pragma unroll
      for (int i = 1; i < 4; ++i) {
        const float4 p = part[i][t][lane];
        o.x += p.x; o.y += p.y; o.z += p.z; o.w += p.w;
      }
      store(t, o);
    }
  }
}

template <int RT>
static void launch_head_linear(const HeadLinearArgs& a, hipStream_t s) {
  const unsigned tiles = (unsigned)((a.rows + 16 * RT - 1) / (16 * RT)), heads = (unsigned)a.heads;
  if (a.K >= 256) head_linear_bf16_kernel<RT, true><<<dim3((unsigned)(a.N / 16), heads, tiles), dim3(256), 0, s>>>(a);
  else head_linear_bf16_kernel<RT, false><<<dim3((unsigned)((a.N + 63) / 64), heads, tiles), dim3(256), 0, s>>>(a);
}

__global__ __launch_bounds__(256) void head_linear_f32_kernel(const HeadLinearArgs a) {
  constexpr int kStep = 64;
  __shared__ float xs[16][kStep + 1], ws[16][kStep + 1];
  const int r = threadIdx.x >> 4, c = threadIdx.x & 15, h = blockIdx.y;
  const int row = blockIdx.z * 16 + r, col = blockIdx.x * 16 + c;
  const float* x = reinterpret_cast<const float*>(a.x) + (int64_t)h * a.x_head;
  const float* w = reinterpret_cast<const float*>(a.w) + (int64_t)h * a.N * a.K;
  float acc = 0.f;
  for (int k0 = 0; k0 < a.K; k0 += kStep) {
    for (int i = threadIdx.x; i < 16 * kStep; i += 256) {
      const int rr = i / kStep, k = i % kStep;
      const int xr = blockIdx.z * 16 + rr, wr = blockIdx.x * 16 + rr;
      xs[rr][k] = xr < a.rows && k0 + k < a.K ? x[(int64_t)xr * a.x_row + k0 + k] : 0.f;
      ws[rr][k] = wr < a.N && k0 + k < a.K ? w[(int64_t)wr * a.K + k0 + k] : 0.f;
    }
    __syncthreads();
#pragma unroll 16
    for (int k = 0; k < kStep; ++k) acc = fmaf(xs[r][k], ws[c][k], acc);
    __syncthreads();
  }
  if (row < a.rows && col < a.N) reinterpret_cast<float*>(a.out)[(int64_t)row * a.out_row + (int64_t)h * a.out_head + col] = acc;
}

}  // namespace mvllm

using namespace mvllm;

extern "C" int mvllm_latent_norm_store(void* out, const void* in, int64_t in_row_stride, const float* weight, float eps,
                                       void* cache, int64_t num_slots, const int64_t* slots, int64_t rows, int rank,
                                       int padded, int dtype, void* stream) {
  const int esize = dtype_size(dtype);
  if (esize == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || rank <= 0 || padded < rank || padded % 32 != 0 || in_row_stride < padded) return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || padded > 2048 || rows > (1 << 30) || (in_row_stride * esize) % 16 != 0) return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0) return MVLLM_OK;
  if (!in || !weight || (!out && !cache) || (cache && !slots)) return MVLLM_ERR_NULL_POINTER;
  if (!aligned16(in) || !aligned16(out) || !aligned16(cache)) return MVLLM_ERR_MISALIGNED;
  LatentNormArgs a = {};
  a.out = out; a.in = in; a.weight = weight; a.cache = cache; a.slots = slots; a.in_stride = in_row_stride;
  a.num_slots = num_slots; a.eps = eps; a.rows = (int)rows; a.rank = rank; a.padded = padded; a.vec = aligned16(weight);
  if (dtype == MVLLM_F32) launch_latent_norm<float>(a, a, false, (hipStream_t)stream);
  else launch_latent_norm<bf16_t>(a, a, false, (hipStream_t)stream);
  return launch_status();
}

extern "C" int mvllm_latent_rope_store(void* out, const int64_t* out_rows, const void* in, int64_t in_row_stride,
                                       const float* weight, float eps, const float* rot_table, int rot_col, int rot,
                                       int rot_dims, int interleaved, int64_t max_position, const int64_t* positions,
                                       void* cache, int64_t num_slots, const int64_t* slots, void* out2, const void* in2,
                                       int64_t in2_row_stride, const float* weight2, int rank2, int padded2, int64_t rows,
                                       int rank, int padded, int dtype, void* stream) {
  const int esize = dtype_size(dtype);
  if (esize == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || rank <= 0 || padded < rank || padded % 32 != 0 || in_row_stride < padded || rot < 0 || rot_dims < 0 || rot_dims > rot ||
      rot_dims % 2 != 0 || (rot > 0 && (rot_col < rank || rot_col % 8 != 0 || rot_col + rot > padded || max_position <= 0)) ||
      (in2 && (rank2 <= 0 || padded2 < rank2 || padded2 % 32 != 0 || in2_row_stride < padded2)))
    return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || padded > 2048 || padded2 > 2048 || rows > (1 << 30) || (in_row_stride * esize) % 16 != 0 || (in2_row_stride * esize) % 16 != 0)
    return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0) return MVLLM_OK;
  if (!in || !weight || (cache && !slots) || (rot > 0 && (!rot_table || !positions)) || (in2 && (!weight2 || !out2))) return MVLLM_ERR_NULL_POINTER;
  if (!aligned16(in) || !aligned16(out) || !aligned16(cache) || !aligned16(in2) || !aligned16(out2)) return MVLLM_ERR_MISALIGNED;
  LatentNormArgs a = {}, b = {};
  a.out = out; a.out_rows = out_rows; a.in = in; a.weight = weight; a.cache = cache; a.slots = slots;
  a.rot_table = rot > 0 ? reinterpret_cast<const float2*>(rot_table) : nullptr; a.positions = positions; a.in_stride = in_row_stride;
  a.num_slots = num_slots; a.max_position = max_position; a.eps = eps; a.rows = (int)rows; a.rank = rank; a.padded = padded;
  a.rot_col = rot_col; a.rot = rot; a.rot_dims = rot_dims; a.interleaved = interleaved; a.vec = aligned16(weight);
  b.out = out2; b.in = in2; b.weight = weight2; b.in_stride = in2_row_stride; b.eps = eps; b.rows = (int)rows; b.rank = rank2;
  b.padded = padded2; b.vec = aligned16(weight2);
  if (dtype == MVLLM_F32) launch_latent_norm<float>(a, b, in2 != nullptr, (hipStream_t)stream);
  else launch_latent_norm<bf16_t>(a, b, in2 != nullptr, (hipStream_t)stream);
  return launch_status();
}

extern "C" int mvllm_head_linear(void* out, int64_t out_row_stride, int64_t out_head_stride, const void* x,
                                 int64_t x_row_stride, int64_t x_head_stride, const void* w, int64_t rows, int num_heads,
                                 int N, int K, int dtype, void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || num_heads <= 0 || N <= 0 || K <= 0 || x_head_stride < K || out_head_stride < N) return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || num_heads > 65535 || rows > 65535 * 16) return MVLLM_ERR_UNSUPPORTED;
  if (dtype == MVLLM_BF16 && (K % 8 != 0 || N % 16 != 0 || x_row_stride % 8 != 0 || x_head_stride % 8 != 0 || out_row_stride % 4 != 0 ||
                              out_head_stride % 4 != 0))
    return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0) return MVLLM_OK;
  if (!out || !x || !w) return MVLLM_ERR_NULL_POINTER;
  if (dtype == MVLLM_BF16 && (!aligned16(x) || !aligned16(w) || (reinterpret_cast<uintptr_t>(out) & 7u) != 0)) return MVLLM_ERR_MISALIGNED;
  HeadLinearArgs a;
  a.out = out; a.x = x; a.w = w; a.out_row = out_row_stride; a.out_head = out_head_stride; a.x_row = x_row_stride;
  a.x_head = x_head_stride; a.rows = (int)rows; a.heads = num_heads; a.N = N; a.K = K;
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MVLLM_F32) head_linear_f32_kernel<<<dim3((unsigned)((N + 15) / 16), (unsigned)num_heads, (unsigned)((rows + 15) / 16)), dim3(256), 0, s>>>(a);
  else if (rows <= 16) launch_head_linear<1>(a, s);
  else if (rows <= 32) launch_head_linear<2>(a, s);
  else launch_head_linear<4>(a, s);
  return launch_status();
}

extern "C" size_t mvllm_latent_decode_workspace_bytes(int rows, int num_heads, int padded, int64_t max_keys, int dtype) {
  if (rows <= 0 || num_heads <= 0 || padded <= 0 || max_keys <= 0) return 0;
  const int parts = plan_parts(rows, num_heads, 1, padded, max_keys, dtype);
  return parts == 1 ? 0 : (size_t)rows * parts * num_heads * ((size_t)padded + 2) * sizeof(float);
}

extern "C" int mvllm_latent_decode(void* out, const void* q, const void* cache, const int32_t* block_tables, int table_width,
                                   const int32_t* row_entry, const int64_t* lens, int rows, int num_heads, int padded,
                                   int block_size, int64_t num_blocks, float scale, int dtype, void* workspace,
                                   size_t workspace_bytes, void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || num_heads <= 0 || padded <= 0 || padded % 32 != 0 || table_width <= 0 || block_size <= 0 || num_blocks <= 0 ||
      (int64_t)table_width * block_size >= (int64_t)1 << 31)
    return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || padded > 2048 || num_heads > 65535 || rows > 65535) return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0) return MVLLM_OK;
  if (!out || !q || !cache || !block_tables || !row_entry || !lens) return MVLLM_ERR_NULL_POINTER;
  if (!aligned16(out) || !aligned16(q) || !aligned16(cache)) return MVLLM_ERR_MISALIGNED;
  LatentDecodeArgs a = {};
  a.out = out; a.q = q; a.cache = cache; a.tables = block_tables; a.row_entry = row_entry; a.lens = lens;
  a.num_blocks = num_blocks; a.table_width = table_width; a.block_size = block_size; a.heads = num_heads; a.padded = padded;
  a.kv_heads = 1; a.values = a.row = padded; a.q_head = a.out_head = padded; a.q_row = a.out_row = (int64_t)num_heads * padded;
  a.scale_log2 = scale * kLog2e;
  a.parts = plan_parts(rows, num_heads, 1, padded, (int64_t)table_width * block_size, dtype);
  a.part_o = nullptr;
  a.part_ml = nullptr;
  if (a.parts > 1) {
    if (!workspace || !aligned16(workspace) || workspace_bytes < mvllm_latent_decode_workspace_bytes(rows, num_heads, padded, (int64_t)table_width * block_size, dtype))
      return MVLLM_ERR_WORKSPACE;
    a.part_o = reinterpret_cast<float*>(workspace);
    a.part_ml = reinterpret_cast<float2*>(a.part_o + (int64_t)rows * a.parts * num_heads * padded);
  }
  return launch_decode<false>(a, rows, dtype, (hipStream_t)stream);
}
