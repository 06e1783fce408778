// The per-head work on both sides of attention for decoders whose heads differ from the q/k-norm + half-split rotary
// form of qk_norm_rope_store.hip: separate q and k norms (or none), a rotary embedding of the first `rot` dims in either
// pair layout with any table of angles, rotated values, key and value sizes that differ, and on the way out the inverse
// rotation of the values and a gate per head.
//
// mvllm_head_rope_store: packed projection rows [q | k | v] ->
//     q_out[dst]  = rotate(rms(q) * gq, pos) * q_scale            [*, H, D]
//     k           = rotate(rms(k) * gk, pos)                      [*, G, D]   packed (k_out) and / or cache slot
//     v           = rotate(v, pos) with a table of its own        [*, G, D]   packed (v_out) and / or cache slot
//   D >= max(dim, vdim) is the head size the attention kernels run at: dims past dim / vdim are written as zeros.
//   dst = dst_row[t] (null: t) reorders the rows for attention, which runs over groups of rows.
// mvllm_head_unrotate_gate: attention output rows [*, H, D] ->
//     out[t, h * vdim + d] = rotate(o[dst_row[t], h], -pos)[d] * sigmoid(gate[t, h])
// Sixteen lanes own one head vector, eight consecutive dims per lane and step; everything is computed in fp32 from the
// loaded values and rounded once.
#include "common.h"

#pragma clang fp contract(off)

namespace mvllm {

constexpr int kLanes = 16;       // lanes per head vector
constexpr int kMaxSteps = 4;     // 8 dims per lane and step: head sizes up to 512

// n (1 .. 8) consecutive values as fp32, zeros behind them; one 16-byte access where the address and n allow it
template <typename T> __device__ __forceinline__ void load8(const T* p, int n, float* v) {
  if (n == 8 && (reinterpret_cast<uintptr_t>(p) & 15u) == 0) {
    if constexpr (sizeof(T) == 4) {
      const float4 a = reinterpret_cast<const float4*>(p)[0], b = reinterpret_cast<const float4*>(p)[1];
      v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
    } else {
      const uint4 w = *reinterpret_cast<const uint4*>(p);
      const uint32_t q[4] = {w.x, w.y, w.z, w.w};
#pragma unroll
      for (int i = 0; i < 4; ++i) { v[2 * i] = lo_to_float<T>(q[i]); v[2 * i + 1] = hi_to_float<T>(q[i]); }
    }
    return;
  }
#pragma unroll
  for (int i = 0; i < 8; ++i) v[i] = i < n ? to_float(p[i]) : 0.f;
}
template <typename T> __device__ __forceinline__ void store8(T* p, int n, const float* v) {
  T r[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) r[i] = from_float<T>(v[i]);
  if (n == 8 && (reinterpret_cast<uintptr_t>(p) & 15u) == 0) {
#pragma unroll
    for (int i = 0; i < (int)(sizeof(r) / 16); ++i) reinterpret_cast<uint4*>(p)[i] = reinterpret_cast<const uint4*>(r)[i];
    return;
  }
#pragma unroll
  for (int i = 0; i < 8; ++i)
    if (i < n) p[i] = r[i];
}

// Rotation of one lane's eight dims d0 .. d0 + 7.  cs: this position's (cos, sin) pairs, rot / 2 of them; `partner` holds
// the eight dims of the other half (half-split layout only, where dim m pairs with m + rot / 2).
__device__ __forceinline__ void rotate8(float* x, const float* partner, int d0, int rot, bool interleaved,
                                        const float2* cs, float sign) {
  if (interleaved) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if (d0 + 2 * i < rot) {
        const float2 c = cs[d0 / 2 + i];
        const float s = c.y * sign, u = x[2 * i], v = x[2 * i + 1];
        x[2 * i] = u * c.x - v * s;
        x[2 * i + 1] = v * c.x + u * s;
      }
    }
  } else {
    const int half = rot / 2;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int d = d0 + i;
      if (d < rot) {
        const bool low = d < half;
        const float2 c = cs[low ? d : d - half];
        x[i] = low ? x[i] * c.x - partner[i] * (c.y * sign) : x[i] * c.x + partner[i] * (c.y * sign);
      }
    }
  }
}

// The half-split partner of dims d0 .. d0 + 7 (element by element: rot / 2 need not be a multiple of 8).
template <typename T> __device__ __forceinline__ void load_partner(const T* row, const float* gain, float scale, int d0, int rot, float* v) {
  const int half = rot / 2;
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const int d = d0 + i;
    v[i] = 0.f;
    if (d < rot) {
      const int p = d < half ? d + half : d - half;
      v[i] = to_float(row[p]) * scale * (gain ? gain[p] : 1.f);
    }
  }
}

struct HeadRopeArgs {
  void* q_out;             // [*, H, D]
  void* k_out;             // [*, G, D] or null
  void* v_out;
  const void* proj;        // [T, proj_stride]: q at 0, k at H dim, v at (H + G) dim
  const float* gain_q;     // [dim] or null (no norm)
  const float* gain_k;
  const float2* rot_table;    // [max_position, rot / 2] (cos, sin) or null
  const float2* v_table;      // [max_position, vdim / 2] or null
  const int64_t* positions;   // [T]
  const int32_t* dst_row;     // [T] or null
  const int64_t* slots;       // [T] or null
  void* k_cache;              // [slots, G, D]
  void* v_cache;
  int64_t proj_stride;
  int64_t max_position;
  int64_t num_slots;
  int64_t rows;
  int heads, kv_heads, dim, vdim, D, rot;
  int interleaved;
  float eps, q_scale;
};

template <typename T>
__global__ __launch_bounds__(256) void head_rope_store_kernel(const HeadRopeArgs a) {
  const int per_row = a.heads + 2 * a.kv_heads;
  const int64_t item = (int64_t)blockIdx.x * (256 / kLanes) + threadIdx.x / kLanes;
  const int li = threadIdx.x % kLanes;
  const bool live = item < a.rows * per_row;
  const int64_t t = live ? item / per_row : 0;
  const int u = live ? (int)(item - t * per_row) : 0;
  const bool is_q = u < a.heads, is_v = u >= a.heads + a.kv_heads;
  const int head = is_q ? u : is_v ? u - a.heads - a.kv_heads : u - a.heads;
  const int n = is_v ? a.vdim : a.dim;
  const T* src = reinterpret_cast<const T*>(a.proj) + t * a.proj_stride +
                 (is_q ? (int64_t)head * a.dim
                       : is_v ? (int64_t)(a.heads + a.kv_heads) * a.dim + (int64_t)head * a.vdim
                              : (int64_t)(a.heads + head) * a.dim);
  const float* gain = is_q ? a.gain_q : is_v ? nullptr : a.gain_k;
  float x[kMaxSteps][8];
  float ss = 0.f;
#pragma unroll
  for (int s = 0; s < kMaxSteps; ++s) {
    const int d0 = 8 * (li + kLanes * s);
#pragma unroll
    for (int i = 0; i < 8; ++i) x[s][i] = 0.f;
    if (live && d0 < n) load8(src + d0, min(8, n - d0), x[s]);
#pragma unroll
    for (int i = 0; i < 8; ++i) ss = fmaf(x[s][i], x[s][i], ss);
  }
#pragma unroll
  for (int o = 1; o < kLanes; o <<= 1) ss += __shfl_xor(ss, o, 64);
  if (!live) return;
  const float scale = gain ? 1.0f / sqrtf(ss / (float)n + a.eps) : 1.0f;
  int64_t pos = a.positions[t];
  pos = pos < 0 ? 0 : pos >= a.max_position ? a.max_position - 1 : pos;
  const int rot = is_v ? (a.v_table ? a.vdim : 0) : (a.rot_table ? a.rot : 0);
  const float2* cs = rot == 0 ? nullptr : (is_v ? a.v_table : a.rot_table) + pos * (rot / 2);
  const int64_t dst = a.dst_row ? a.dst_row[t] : t;
  const int64_t slot = !is_q && a.slots ? a.slots[t] : -1;
  T* packed = reinterpret_cast<T*>(is_q ? a.q_out : is_v ? a.v_out : a.k_out);
  const int groups = is_q ? a.heads : a.kv_heads;
  if (packed) packed += (dst * groups + head) * a.D;
  T* cached = nullptr;
  if (slot >= 0 && slot < a.num_slots) cached = reinterpret_cast<T*>(is_v ? a.v_cache : a.k_cache) + (slot * a.kv_heads + head) * a.D;
#pragma unroll
  for (int s = 0; s < kMaxSteps; ++s) {
    const int d0 = 8 * (li + kLanes * s);
    if (d0 >= a.D) continue;
    if (gain) {
#pragma unroll
      for (int i = 0; i < 8; ++i) x[s][i] = d0 + i < n ? x[s][i] * scale * gain[d0 + i] : 0.f;
    }
    if (d0 < rot) {
      float partner[8];
      if (!a.interleaved) load_partner(src, gain, scale, d0, rot, partner);
      rotate8(x[s], partner, d0, rot, a.interleaved != 0, cs, 1.f);
    }
    if (is_q) {
#pragma unroll
      for (int i = 0; i < 8; ++i) x[s][i] *= a.q_scale;
    }
    const int m = min(8, a.D - d0);
    if (packed) store8(packed + d0, m, x[s]);
    if (cached) store8(cached + d0, m, x[s]);
  }
}

struct UnrotateGateArgs {
  void* out;                  // [T, H * vdim]
  const void* o;              // [*, H, D]
  const void* gate;           // [T, gate_stride], H values per row, or null
  const float2* v_table;      // [max_position, vdim / 2] or null
  const int64_t* positions;
  const int32_t* dst_row;     // [T] or null
  int64_t gate_stride;
  int64_t max_position;
  int64_t rows;
  int heads, vdim, D;
  int interleaved;
};

template <typename T>
__global__ __launch_bounds__(256) void head_unrotate_gate_kernel(const UnrotateGateArgs a) {
  const int64_t item = (int64_t)blockIdx.x * (256 / kLanes) + threadIdx.x / kLanes;
  const int li = threadIdx.x % kLanes;
  if (item >= a.rows * a.heads) return;
  const int64_t t = item / a.heads;
  const int h = (int)(item - t * a.heads);
  const int64_t src_row = a.dst_row ? a.dst_row[t] : t;
  const T* src = reinterpret_cast<const T*>(a.o) + (src_row * a.heads + h) * a.D;
  T* dst = reinterpret_cast<T*>(a.out) + (t * a.heads + h) * a.vdim;
  float g = 1.f;
  if (a.gate) g = 1.0f / (1.0f + __expf(-to_float(reinterpret_cast<const T*>(a.gate)[t * a.gate_stride + h])));
  int64_t pos = a.positions[t];
  pos = pos < 0 ? 0 : pos >= a.max_position ? a.max_position - 1 : pos;
  const int rot = a.v_table ? a.vdim : 0;
  const float2* cs = rot ? a.v_table + pos * (rot / 2) : nullptr;
#pragma unroll
  for (int s = 0; s < kMaxSteps; ++s) {
    const int d0 = 8 * (li + kLanes * s);
    if (d0 >= a.vdim) continue;
    const int n = min(8, a.vdim - d0);
    float x[8];
    load8(src + d0, n, x);
    if (d0 < rot) {
      float partner[8];
      if (!a.interleaved) load_partner(src, nullptr, 1.f, d0, rot, partner);
      rotate8(x, partner, d0, rot, a.interleaved != 0, cs, -1.f);
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) x[i] *= g;
    store8(dst + d0, n, x);
  }
}

// Where a decode row's token lies in a cache that holds one attention chunk per sequence: context length inside the
// chunk and the slot its key and value go to.  One thread per row; rows with a context of 0 (padding) store nothing.
__global__ __launch_bounds__(256) void chunk_decode_step_kernel(int64_t* chunk_lens, int64_t* slots, const int64_t* context_lens,
                                                                const int32_t* tables, int table_width, int chunk, int block_size,
                                                                int batch) {
  const int b = blockIdx.x * 256 + threadIdx.x;
  if (b >= batch) return;
  const int64_t ctx = context_lens[b];
  int64_t len = 0, slot = -1;
  if (ctx > 0) {
    const int64_t at = chunk > 0 ? (ctx - 1) % chunk : ctx - 1;
    const int64_t bi = at / block_size;
    const int phys = bi < table_width ? tables[(int64_t)b * table_width + bi] : -1;
    len = at + 1;
    if (phys >= 0) slot = (int64_t)phys * block_size + at % block_size;
  }
  chunk_lens[b] = len;
  slots[b] = slot;
}

}  // namespace mvllm

using namespace mvllm;

static unsigned head_blocks(int64_t items) { return (unsigned)((items + 256 / kLanes - 1) / (256 / kLanes)); }

extern "C" int mvllm_head_rope_store(void* q_out, void* k_out, void* v_out, const void* proj, int64_t proj_row_stride,
                                     const float* gain_q, const float* gain_k, float eps, float q_scale,
                                     const float* rot_table, int rot_dims, const float* v_table, int interleaved,
                                     int64_t max_position, const int64_t* positions, const int32_t* dst_row,
                                     const int64_t* slots, void* k_cache, void* v_cache, int64_t num_slots, int64_t rows,
                                     int num_heads, int num_kv_heads, int dim, int vdim, int head_dim, int dtype,
                                     void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || num_heads <= 0 || num_kv_heads <= 0 || num_heads % num_kv_heads != 0 || dim <= 0 || vdim <= 0 ||
      head_dim < dim || head_dim < vdim || rot_dims < 0 || rot_dims > dim || rot_dims % 2 != 0 ||
      (v_table && vdim % 2 != 0) || max_position <= 0 || num_slots < 0 ||
      proj_row_stride < (int64_t)num_heads * dim + (int64_t)num_kv_heads * (dim + vdim))
    return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || head_dim > 8 * kLanes * kMaxSteps) return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0) return MVLLM_OK;
  if (!q_out || !proj || !positions || (slots && (!k_cache || !v_cache)) || (rot_dims && !rot_table)) return MVLLM_ERR_NULL_POINTER;
  HeadRopeArgs a;
  a.q_out = q_out; a.k_out = k_out; a.v_out = v_out; a.proj = proj; a.gain_q = gain_q; a.gain_k = gain_k;
  a.rot_table = rot_dims ? reinterpret_cast<const float2*>(rot_table) : nullptr;
  a.v_table = reinterpret_cast<const float2*>(v_table);
  a.positions = positions; a.dst_row = dst_row; a.slots = slots; a.k_cache = k_cache; a.v_cache = v_cache;
  a.proj_stride = proj_row_stride; a.max_position = max_position; a.num_slots = num_slots; a.rows = rows;
  a.heads = num_heads; a.kv_heads = num_kv_heads; a.dim = dim; a.vdim = vdim; a.D = head_dim; a.rot = rot_dims;
  a.interleaved = interleaved; a.eps = eps; a.q_scale = q_scale;
  const unsigned grid = head_blocks(rows * (num_heads + 2 * (int64_t)num_kv_heads));
  if (dtype == MVLLM_F32) head_rope_store_kernel<float><<<dim3(grid), dim3(256), 0, (hipStream_t)stream>>>(a);
  else head_rope_store_kernel<bf16_t><<<dim3(grid), dim3(256), 0, (hipStream_t)stream>>>(a);
  return launch_status();
}

extern "C" int mvllm_head_unrotate_gate(void* out, const void* o, const void* gate, int64_t gate_row_stride,
                                        const float* v_table, int interleaved, int64_t max_position,
                                        const int64_t* positions, const int32_t* dst_row, int64_t rows, int num_heads,
                                        int vdim, int head_dim, int dtype, void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || num_heads <= 0 || vdim <= 0 || head_dim < vdim || (v_table && vdim % 2 != 0) || max_position <= 0 ||
      (gate && gate_row_stride < num_heads))
    return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || head_dim > 8 * kLanes * kMaxSteps) return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0) return MVLLM_OK;
  if (!out || !o || !positions) return MVLLM_ERR_NULL_POINTER;
  UnrotateGateArgs a;
  a.out = out; a.o = o; a.gate = gate; a.v_table = reinterpret_cast<const float2*>(v_table); a.positions = positions;
  a.dst_row = dst_row; a.gate_stride = gate_row_stride; a.max_position = max_position; a.rows = rows;
  a.heads = num_heads; a.vdim = vdim; a.D = head_dim; a.interleaved = interleaved;
  const unsigned grid = head_blocks(rows * num_heads);
  if (dtype == MVLLM_F32) head_unrotate_gate_kernel<float><<<dim3(grid), dim3(256), 0, (hipStream_t)stream>>>(a);
  else head_unrotate_gate_kernel<bf16_t><<<dim3(grid), dim3(256), 0, (hipStream_t)stream>>>(a);
  return launch_status();
}

extern "C" int mvllm_chunk_decode_step(int64_t* chunk_lens, int64_t* slots, const int64_t* context_lens,
                                       const int32_t* block_tables, int max_num_blocks, int chunk, int block_size,
                                       int batch, void* stream) {
  if (batch < 0 || max_num_blocks <= 0 || chunk < 0 || block_size <= 0) return MVLLM_ERR_BAD_SHAPE;
  if (batch == 0) return MVLLM_OK;
  if (!chunk_lens || !slots || !context_lens || !block_tables) return MVLLM_ERR_NULL_POINTER;
  chunk_decode_step_kernel<<<dim3((unsigned)((batch + 255) / 256)), dim3(256), 0, (hipStream_t)stream>>>(
      chunk_lens, slots, context_lens, block_tables, max_num_blocks, chunk, block_size, batch);
  return launch_status();
}
