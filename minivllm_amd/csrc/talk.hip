// Attention with mixed heads (talk.h): entry points, and the kernel for every size and type.
#include "talk.h"

#pragma clang fp contract(off)

namespace mvllm {

constexpr int kAnyKeys = 64, kAnyHeads = 64;

// Any size with at most 64 heads and 256 NE output columns: a workgroup is a query row with all its heads, 64 keys at a time.
// Sixteen lanes make a key's raw scores for the heads of a kv head, a lane is a key where heads are mixed and weighed, a
// thread owns output columns.
template <typename T, int NE>
__global__ __launch_bounds__(256) void talk_any_kernel(const TalkArgs a) {
  __shared__ float raw[kAnyHeads][kAnyKeys], weight[kAnyHeads][kAnyKeys];
  __shared__ float top[kAnyHeads], sum[kAnyHeads], keep[kAnyHeads];
  __shared__ int64_t key_row[kAnyKeys];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, li = tid & 15, group = tid >> 4;
  const int H = a.heads, G = a.kv_heads, D = a.dim, per = H / G;
  int64_t t = blockIdx.x;
  int64_t first = 0;
  const int32_t* table = nullptr;
  int keys;
  if (a.cu_q) {
    int seq_start, seq_len, r, seq;
    if (!locate_tile(a.cu_q, a.num_seqs, blockIdx.x, 1, seq_start, seq_len, r, seq)) return;
    t = (int64_t)seq_start + r;
    const int past = a.cu_k ? a.cu_k[seq + 1] - a.cu_k[seq] - seq_len : 0;
    keys = past + r + 1;
    if (a.tables) table = a.tables + (int64_t)seq * a.table_width;
    else first = a.cu_k ? a.cu_k[seq] : seq_start;
  } else {
    table = a.tables + t * a.table_width;
    keys = (int)min(max(a.lens[t], (int64_t)0), (int64_t)a.table_width * a.block_size);
  }
  for (int h = tid; h < H; h += 256) {
    top[h] = -INFINITY;
    sum[h] = 0.f;
  }
  const T* q = reinterpret_cast<const T*>(a.q) + t * H * D;
  float o[NE];
#pragma unroll
  for (int i = 0; i < NE; ++i) o[i] = 0.f;
  for (int base = 0; base < keys; base += kAnyKeys) {
    __syncthreads();
    if (tid < kAnyKeys) {
      const int j = min(base + tid, keys - 1);
      if (table) {
        const int b = j / a.block_size;
        key_row[tid] = min(max((int64_t)table[b], (int64_t)0), a.num_blocks - 1) * a.block_size + (j - b * a.block_size);
      } else {
        key_row[tid] = first + j;
      }
    }
    __syncthreads();
    for (int item = group; item < kAnyKeys * G; item += 16) {
      const int j = item % kAnyKeys, kv = item / kAnyKeys;
      const T* k = reinterpret_cast<const T*>(a.k) + (key_row[j] * G + kv) * D;
      for (int h = kv * per; h < (kv + 1) * per; ++h) {
        float s = 0.f;
        for (int d = li; d < D; d += 16) s = fmaf(to_float(q[h * D + d]), to_float(k[d]), s);
        s = row16_sum(s);
        if (li == 0) raw[h][j] = s;
      }
    }
    __syncthreads();
    for (int h = wave; h < H; h += 4) {
      float s = 0.f;
      for (int g = 0; g < H; ++g) s = fmaf(a.talk[h * H + g], raw[g][lane], s);
      if (base + lane >= keys) s = -INFINITY;
      const float m = top[h], m_new = fmaxf(m, wave_max(s)), p = exp2f(s - m_new), l = wave_sum(p);
      weight[h][lane] = p;
      if (lane == 0) {
        keep[h] = exp2f(m - m_new);
        top[h] = m_new;
        sum[h] = sum[h] * keep[h] + l;
      }
    }
    __syncthreads();
    const int n = min(kAnyKeys, keys - base);
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int c = tid + 256 * i;
      if (c >= H * D) continue;
      const int h = c / D;
      const T* v = reinterpret_cast<const T*>(a.v) + (int64_t)(h / per) * D + (c - h * D);
      float x = o[i] * keep[h];
      for (int j = 0; j < n; ++j) x = fmaf(weight[h][j], to_float(v[key_row[j] * G * D]), x);
      o[i] = x;
    }
  }
  __syncthreads();
  T* out = reinterpret_cast<T*>(a.out) + (a.out_rows ? (int64_t)a.out_rows[t] : t) * a.out_row;
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int c = tid + 256 * i;
    if (c >= H * D) continue;
    const int h = c / D;
    float l = sum[h];
    if (a.sinks && l > 0.f) l += exp2f(a.sinks[h] * kLog2e - top[h]);
    out[h * a.out_head + (c - h * D)] = from_float<T>(l > 0.f ? o[i] / l : 0.f);
  }
}

template <typename T>
static int launch_talk_any(const TalkArgs& a, int64_t rows, hipStream_t s) {
  const int64_t columns = (int64_t)a.heads * a.dim;
  if (a.heads > kAnyHeads || columns > 16384) return MVLLM_ERR_UNSUPPORTED;
  const dim3 grid((unsigned)rows), block(256);
  if (columns <= 1024) talk_any_kernel<T, 4><<<grid, block, 0, s>>>(a);
  else if (columns <= 4096) talk_any_kernel<T, 16><<<grid, block, 0, s>>>(a);
  else talk_any_kernel<T, 64><<<grid, block, 0, s>>>(a);
  return launch_status();
}

__attribute__((weak)) int launch_talk_prefill(const TalkArgs&, hipStream_t) { return kNotBuilt; }
__attribute__((weak)) int launch_talk_decode(const TalkArgs&, int, hipStream_t) { return kNotBuilt; }

// Whether the tiled kernels are built for the heads, whatever the number of rows.
static bool talk_tiles(int heads, int kv_heads, int dim, int dtype) {
  return dtype == MVLLM_BF16 && heads <= 64 && heads / kv_heads <= 32 && kv_heads <= 8 && (dim == 32 || dim == 64 || dim == 96 || dim == 128);
}

// Shares of a decoded row, as plan_parts: a workgroup takes all heads of its share, two run on a CU.
static int talk_parts(int rows, int heads, int kv_heads, int dim, int64_t max_keys, int dtype) {
  if (!talk_tiles(heads, kv_heads, dim, dtype)) return 1;
  const int64_t tiles = (max_keys + 63) / 64, together = 512;
  int best = 1;
  int64_t best_time = INT64_MAX;
  for (int parts = 1; parts <= kMaxParts && (parts == 1 || 2 * parts <= tiles); ++parts) {
    const int64_t time = ((int64_t)rows * parts + together - 1) / together * ((tiles + parts - 1) / parts + 2) + (parts > 1 ? 2 : 0);
    if (time < best_time) {
      best = parts;
      best_time = time;
    }
  }
  return best;
}

}  // namespace mvllm

using namespace mvllm;

static int talk_check(const void* out, int64_t out_row, int64_t out_head, const void* q, const void* k, const void* v, const float* talk,
                      int64_t rows, int heads, int kv_heads, int dim, int dtype) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || heads <= 0 || kv_heads <= 0 || heads % kv_heads != 0 || dim <= 0 || dim % 8 != 0 || out_head < dim || out_row < 0 ||
      out_row % 4 != 0 || out_head % 4 != 0)
    return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || heads > kAnyHeads || (int64_t)heads * dim > 16384 || rows > ((int64_t)1 << 30)) return MVLLM_ERR_UNSUPPORTED;
  if (rows > 0 && (!out || !q || !k || !v || !talk)) return MVLLM_ERR_NULL_POINTER;
  if (!aligned16(out) || !aligned16(q) || !aligned16(k) || !aligned16(v)) return MVLLM_ERR_MISALIGNED;
  return MVLLM_OK;
}

extern "C" int mvllm_talk_prefill(void* out, int64_t out_row_stride, int64_t out_head_stride, const int32_t* out_rows, const void* q,
                                  const void* k, const void* v, const int32_t* cu_q, const int32_t* cu_k,
                                  const int32_t* block_tables, int table_width, int block_size, int64_t num_blocks,
                                  const float* talk, const float* sinks, int num_seqs, int64_t total_q, int num_heads,
                                  int num_kv_heads, int dim, int dtype, void* stream) {
  const int st = talk_check(out, out_row_stride, out_head_stride, q, k, v, talk, total_q, num_heads, num_kv_heads, dim, dtype);
  if (st != MVLLM_OK) return st;
  if (num_seqs < 0 || (block_tables && (!cu_k || table_width <= 0 || block_size <= 0 || num_blocks <= 0 ||
                                        (int64_t)table_width * block_size >= (int64_t)1 << 31 || num_blocks * block_size >= (int64_t)1 << 31)))
    return MVLLM_ERR_BAD_SHAPE;
  if (num_seqs == 0 || total_q == 0) return MVLLM_OK;
  if (!cu_q) return MVLLM_ERR_NULL_POINTER;
  TalkArgs a = {};
  a.out = out; a.out_row = out_row_stride; a.out_head = out_head_stride; a.out_rows = out_rows; a.q = q; a.k = k; a.v = v;
  a.cu_q = cu_q; a.cu_k = cu_k; a.tables = block_tables; a.table_width = table_width; a.block_size = block_size;
  a.num_blocks = num_blocks; a.talk = talk; a.sinks = sinks; a.num_seqs = num_seqs; a.total_q = total_q; a.heads = num_heads;
  a.kv_heads = num_kv_heads; a.dim = dim; a.parts = 1;
  hipStream_t s = (hipStream_t)stream;
  if (talk_tiles(num_heads, num_kv_heads, dim, dtype) && (!block_tables || block_size % 16 == 0)) {
    const int tiled = launch_talk_prefill(a, s);
    if (tiled != kNotBuilt) return tiled;
  }
  return dtype == MVLLM_F32 ? launch_talk_any<float>(a, total_q, s) : launch_talk_any<bf16_t>(a, total_q, s);
}

extern "C" size_t mvllm_talk_decode_workspace_bytes(int rows, int num_heads, int num_kv_heads, int dim, int64_t max_keys, int dtype) {
  if (rows <= 0 || num_heads <= 0 || num_kv_heads <= 0 || dim <= 0 || max_keys <= 0) return 0;
  const int parts = talk_parts(rows, num_heads, num_kv_heads, dim, max_keys, dtype);
  return parts == 1 ? 0 : (size_t)rows * parts * num_heads * ((size_t)dim + 2) * sizeof(float);
}

extern "C" int mvllm_talk_decode(void* out, int64_t out_row_stride, int64_t out_head_stride, const void* q, const void* k_cache,
                                 const void* v_cache, const int32_t* block_tables, int table_width, const int64_t* lens,
                                 const float* talk, const float* sinks, int rows, int num_heads, int num_kv_heads, int dim,
                                 int block_size, int64_t num_blocks, int dtype, void* workspace, size_t workspace_bytes,
                                 void* stream) {
  const int st = talk_check(out, out_row_stride, out_head_stride, q, k_cache, v_cache, talk, rows, num_heads, num_kv_heads, dim, dtype);
  if (st != MVLLM_OK) return st;
  if (table_width <= 0 || block_size <= 0 || num_blocks <= 0 || (int64_t)table_width * block_size >= (int64_t)1 << 31 ||
      num_blocks * block_size >= (int64_t)1 << 31)
    return MVLLM_ERR_BAD_SHAPE;
  if (rows > 65535) return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0) return MVLLM_OK;
  if (!block_tables || !lens) return MVLLM_ERR_NULL_POINTER;
  TalkArgs a = {};
  a.out = out; a.out_row = out_row_stride; a.out_head = out_head_stride; a.q = q; a.k = k_cache; a.v = v_cache; a.tables = block_tables;
  a.table_width = table_width; a.lens = lens; a.talk = talk; a.sinks = sinks; a.heads = num_heads; a.kv_heads = num_kv_heads;
  a.dim = dim; a.block_size = block_size; a.num_blocks = num_blocks; a.total_q = rows; a.parts = 1;
  hipStream_t s = (hipStream_t)stream;
  if (talk_tiles(num_heads, num_kv_heads, dim, dtype) && block_size % 16 == 0) {
    const int64_t max_keys = (int64_t)table_width * block_size;
    a.parts = talk_parts(rows, num_heads, num_kv_heads, dim, max_keys, dtype);
    if (a.parts > 1) {
      if (!workspace || !aligned16(workspace) || workspace_bytes < mvllm_talk_decode_workspace_bytes(rows, num_heads, num_kv_heads, dim, max_keys, dtype))
        return MVLLM_ERR_WORKSPACE;
      a.part_o = reinterpret_cast<float*>(workspace);
      a.part_ml = reinterpret_cast<float2*>(a.part_o + (int64_t)rows * a.parts * num_heads * dim);
    }
    const int tiled = launch_talk_decode(a, rows, s);
    if (tiled != kNotBuilt) return tiled;
    a.parts = 1;
  }
  return dtype == MVLLM_F32 ? launch_talk_any<float>(a, rows, s) : launch_talk_any<bf16_t>(a, rows, s);
}
