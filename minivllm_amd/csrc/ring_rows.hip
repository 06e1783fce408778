// Rows on their way to and from windowed attention.
//   copy_rows   rows of one matrix to rows of one or two others, by index: new keys into the ring and in front of the prefill
//               kernel, cached ones out of it
//   head_rope   the rotated part of every query head, where it lies or behind the absorbed query of the first rows
#include "common.h"

#pragma clang fp contract(off)

namespace mvllm {

struct CopyRowsArgs {
  char* dst[2];
  const int64_t* dst_rows[2];    // [rows], < 0: not copied; null: row t
  int64_t dst_stride[2];         // bytes
  int64_t dst_count[2];          // rows of dst
  const char* src;
  const int64_t* src_rows;       // [rows] or null
  int64_t src_stride, src_count;
  int64_t rows;
  int chunks;                    // of 16 bytes per row
};

__global__ __launch_bounds__(256) void copy_rows_kernel(const CopyRowsArgs a) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  const int64_t t = i / a.chunks;
  if (t >= a.rows) return;
  const int64_t at = (i - t * a.chunks) * 16;
  const int64_t from = a.src_rows ? a.src_rows[t] : t;
  int64_t to[2];
#pragma unroll
  for (int d = 0; d < 2; ++d) {
    to[d] = !a.dst[d] ? -1 : a.dst_rows[d] ? a.dst_rows[d][t] : t;
    if (to[d] >= a.dst_count[d]) to[d] = -1;
  }
  if (from < 0 || from >= a.src_count || (to[0] < 0 && to[1] < 0)) return;
  const uint4 v = *reinterpret_cast<const uint4*>(a.src + from * a.src_stride + at);
#pragma unroll
  for (int d = 0; d < 2; ++d)
    if (to[d] >= 0) *reinterpret_cast<uint4*>(a.dst[d] + to[d] * a.dst_stride[d] + at) = v;
}

struct HeadRopeRowsArgs {
  void* x;                       // [rows, H, *]: the rotated part of head h at h * x_head + x_col
  void* first_out;               // the same of the first rows goes here instead, zeros behind it
  const float2* table;           // [max_position, dims / 2] (cos, sin)
  const int64_t* positions;
  int64_t x_row, x_head, out_row, out_head, max_position;
  int rows, first, heads, x_col, out_col, rot, dims, out_width, interleaved, units;
};

// A thread takes kPairs pairs (2 kPairs columns) of a head; units behind the last pair move what does not turn, and zeros.
// kPairs = 8: every part is a multiple of sixteen columns and starts on sixteen bytes.
template <typename T, int kPairs>
__global__ __launch_bounds__(256) void head_rope_rows_kernel(const HeadRopeRowsArgs a) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  const int64_t item = i / a.units;
  const int u = (int)(i - item * a.units);
  const int64_t row = item / a.heads;
  const int h = (int)(item - row * a.heads);
  if (row >= a.rows) return;
  T* x = reinterpret_cast<T*>(a.x) + row * a.x_row + h * a.x_head + a.x_col;
  const bool moved = row < a.first;
  T* out = moved ? reinterpret_cast<T*>(a.first_out) + row * a.out_row + h * a.out_head + a.out_col : x;
  const int half = a.dims / 2, p0 = u * kPairs;
  if (p0 >= half) {                                          // behind the pairs
    if (!moved) return;
    const int c0 = a.dims + 2 * (p0 - half);
#pragma unroll
    for (int j = 0; j < 2 * kPairs; ++j)
      if (c0 + j < a.out_width) out[c0 + j] = c0 + j < a.rot ? x[c0 + j] : from_float<T>(0.f);
    return;
  }
  const float2* cs = a.table + min(max(a.positions[row], (int64_t)0), a.max_position - 1) * half + p0;
  const int lo = a.interleaved ? 2 * p0 : p0, hi = a.interleaved ? lo + 1 : p0 + half;
  T v[2 * kPairs], r[2 * kPairs];                            // low (even) columns of a pair and high (odd) ones, as they lie
  if constexpr (kPairs == 8) {
    constexpr int kWords = 8 * (int)sizeof(T) / 16;
    const T* second = a.interleaved ? x + lo + 8 : x + hi;
#pragma unroll
    for (int w = 0; w < kWords; ++w) {
      reinterpret_cast<uint4*>(v)[w] = reinterpret_cast<const uint4*>(x + lo)[w];
      reinterpret_cast<uint4*>(v + 8)[w] = reinterpret_cast<const uint4*>(second)[w];
    }
  } else {
    v[0] = x[lo];
    v[1] = x[hi];
  }
#pragma unroll
  for (int j = 0; j < kPairs; ++j) {
    const float2 c = cs[j];
    const int iu = kPairs == 8 && !a.interleaved ? j : 2 * j, iv = kPairs == 8 && !a.interleaved ? 8 + j : 2 * j + 1;
    const float p = to_float(v[iu]), q = to_float(v[iv]);
    r[iu] = from_float<T>(p * c.x - q * c.y);
    r[iv] = from_float<T>(q * c.x + p * c.y);
  }
  if constexpr (kPairs == 8) {
    constexpr int kWords = 8 * (int)sizeof(T) / 16;
    T* second = a.interleaved ? out + lo + 8 : out + hi;
#pragma unroll
    for (int w = 0; w < kWords; ++w) {
      reinterpret_cast<uint4*>(out + lo)[w] = reinterpret_cast<const uint4*>(r)[w];
      reinterpret_cast<uint4*>(second)[w] = reinterpret_cast<const uint4*>(r + 8)[w];
    }
  } else {
    out[lo] = r[0];
    out[hi] = r[1];
  }
}

}  // namespace mvllm

using namespace mvllm;

extern "C" int mvllm_copy_rows(void* dst, int64_t dst_row_stride, int64_t dst_count, const int64_t* dst_rows, void* dst2,
                               int64_t dst2_row_stride, int64_t dst2_count, const int64_t* dst2_rows, const void* src,
                               int64_t src_row_stride, int64_t src_count, const int64_t* src_rows, int64_t rows, int width,
                               int dtype, void* stream) {
  const int esize = dtype_size(dtype);
  if (esize == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || width <= 0 || src_row_stride < width || (dst && dst_row_stride < width) || (dst2 && dst2_row_stride < width) ||
      src_count < 0 || dst_count < 0 || dst2_count < 0)
    return MVLLM_ERR_BAD_SHAPE;
  if ((width * esize) % 16 != 0 || (src_row_stride * esize) % 16 != 0 || (dst_row_stride * esize) % 16 != 0 || (dst2_row_stride * esize) % 16 != 0)
    return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0 || (!dst && !dst2)) return MVLLM_OK;
  if (!src) return MVLLM_ERR_NULL_POINTER;
  if (!aligned16(src) || !aligned16(dst) || !aligned16(dst2)) return MVLLM_ERR_MISALIGNED;
  CopyRowsArgs a;
  a.dst[0] = reinterpret_cast<char*>(dst); a.dst[1] = reinterpret_cast<char*>(dst2); a.dst_rows[0] = dst_rows; a.dst_rows[1] = dst2_rows;
  a.dst_stride[0] = dst_row_stride * esize; a.dst_stride[1] = dst2_row_stride * esize; a.dst_count[0] = dst_count; a.dst_count[1] = dst2_count;
  a.src = reinterpret_cast<const char*>(src); a.src_rows = src_rows; a.src_stride = src_row_stride * esize; a.src_count = src_count;
  a.rows = rows; a.chunks = width * esize / 16;
  const int64_t blocks = (rows * a.chunks + 255) / 256;
  if (blocks > 0x7fffffff) return MVLLM_ERR_UNSUPPORTED;
  copy_rows_kernel<<<dim3((unsigned)blocks), dim3(256), 0, (hipStream_t)stream>>>(a);
  return launch_status();
}

extern "C" int mvllm_head_rope(void* x, int64_t x_row_stride, int64_t x_head_stride, int x_col, void* first_out,
                               int64_t out_row_stride, int64_t out_head_stride, int out_col, int out_width, int64_t first_rows,
                               const float* table, int rot, int rot_dims, int interleaved, int64_t max_position,
                               const int64_t* positions, int64_t rows, int num_heads, int dtype, void* stream) {
  const int esize = dtype_size(dtype);
  if (esize == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || first_rows < 0 || first_rows > rows || num_heads <= 0 || rot <= 0 || rot_dims < 0 || rot_dims > rot || rot_dims % 2 != 0 ||
      x_col < 0 || x_head_stride < x_col + rot || max_position <= 0 ||
      (first_rows > 0 && (out_col < 0 || out_width < rot || out_head_stride < out_col + out_width)))
    return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || rows > (1 << 28)) return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0) return MVLLM_OK;
  if (!x || !table || !positions || (first_rows > 0 && !first_out)) return MVLLM_ERR_NULL_POINTER;
  HeadRopeRowsArgs a;
  a.x = x; a.first_out = first_out; a.table = reinterpret_cast<const float2*>(table); a.positions = positions; a.x_row = x_row_stride;
  a.x_head = x_head_stride; a.out_row = out_row_stride; a.out_head = out_head_stride; a.max_position = max_position;
  a.rows = (int)rows; a.first = (int)first_rows; a.heads = num_heads; a.x_col = x_col; a.out_col = out_col; a.rot = rot;
  a.dims = rot_dims; a.out_width = out_width; a.interleaved = interleaved;
  const int per16 = 16 / esize;
  const bool vec = rot_dims % 16 == 0 && aligned16(x) && x_row_stride % per16 == 0 && x_head_stride % per16 == 0 && x_col % per16 == 0 &&
                   (first_rows == 0 || (aligned16(first_out) && out_row_stride % per16 == 0 && out_head_stride % per16 == 0 && out_col % per16 == 0));
  const int pairs = vec ? 8 : 1, behind = first_rows > 0 ? out_width - rot_dims : 0;
  a.units = rot_dims / 2 / pairs + (behind + 2 * pairs - 1) / (2 * pairs);
  if (a.units == 0) return MVLLM_OK;
  const int64_t blocks = (rows * num_heads * a.units + 255) / 256;
  if (blocks > 0x7fffffff) return MVLLM_ERR_UNSUPPORTED;
  const dim3 grid((unsigned)blocks), block(256);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MVLLM_F32) {
    if (vec) head_rope_rows_kernel<float, 8><<<grid, block, 0, s>>>(a);
    else head_rope_rows_kernel<float, 1><<<grid, block, 0, s>>>(a);
  } else {
    if (vec) head_rope_rows_kernel<bf16_t, 8><<<grid, block, 0, s>>>(a);
    else head_rope_rows_kernel<bf16_t, 1><<<grid, block, 0, s>>>(a);
  }
  return launch_status();
}
