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
// mvllm_head_norm_rope_store: the same with other norms: q and k over all heads of a row at once (a workgroup per row),
// q and k divided by their root mean square behind the rotation, values divided by theirs; a factor per query head; packed
// keys and values at rows of their own; any distance between the heads of a key or value row (so that a key and its
// value may be neighbours).
// mvllm_head_unrotate_gate: attention output rows [*, H, D] ->
//     out[t, h * vdim + d] = rotate(o[dst_row[t], h], -pos)[d] * sigmoid(gate[t, h])
// Sixteen lanes own one head vector, eight consecutive dims per lane and step (in long batches four heads of a row, which
// share the row's angles); everything is computed in fp32 from the
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
    for (int i = 0; i < (int)(sizeof(r) / 16); ++i) store16_stream(reinterpret_cast<uint4*>(p) + i, reinterpret_cast<const uint4*>(r)[i]);
    return;
  }
#pragma unroll
  for (int i = 0; i < 8; ++i)
    if (i < n) p[i] = r[i];
}

// (cos, sin) of the four pairs among dims d0 .. d0 + 7 of a row of angles, rot / 2 of them; pairs past the end stay as
// they are.
__device__ __forceinline__ void load_angles(float2* angle, const float2* cs, int d0, int rot) {
  if (d0 + 8 <= rot && (reinterpret_cast<uintptr_t>(cs) & 15u) == 0) {
    const float4 a = reinterpret_cast<const float4*>(cs)[d0 / 4], b = reinterpret_cast<const float4*>(cs)[d0 / 4 + 1];
    angle[0] = make_float2(a.x, a.y); angle[1] = make_float2(a.z, a.w);
    angle[2] = make_float2(b.x, b.y); angle[3] = make_float2(b.z, b.w);
    return;
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) angle[i] = d0 + 2 * i < rot ? cs[d0 / 2 + i] : make_float2(1.f, 0.f);
}

// Rotation of one lane's eight dims, pairs (2i, 2i + 1).
__device__ __forceinline__ void turn_pairs(float* x, const float2* angle, float sign) {
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const float2 c = angle[i];
    const float s = c.y * sign, u = x[2 * i], v = x[2 * i + 1];
    x[2 * i] = u * c.x - v * s;
    x[2 * i + 1] = v * c.x + u * s;
  }
}

// The same for pairs (m, m + rot / 2): `partner` holds the eight dims of the other half.
__device__ __forceinline__ void turn_halves(float* x, const float* partner, int d0, int rot, const float2* cs, float sign) {
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
  const float* gain_q;     // [dim], with kNormRows [H dim], or null (no norm)
  const float* gain_k;     // [dim], with kNormRows [G dim]
  const float* head_scale; // [H] or null: further factor of q
  const float2* rot_table;    // [max_position, rot / 2] (cos, sin) or null
  const float2* v_table;      // [max_position, vdim / 2] or null
  const int64_t* positions;   // [T]
  const int32_t* dst_row;     // [T] or null
  const int64_t* kv_row;      // [T] or null (dst): rows of k_out and v_out, negative: none
  const int64_t* slots;       // [T] or null
  void* k_cache;              // [slots, G, kv_head]: heads in the first D
  void* v_cache;
  int64_t proj_stride;
  int64_t max_position;
  int64_t num_slots;
  int64_t rows;
  int heads, kv_heads, dim, vdim, D, rot;
  int interleaved, norms, kv_head;
  float eps, q_scale;
};

enum { kNormRows = 1, kNormTurned = 2, kNormValues = 4 };
constexpr int kMaxRowParts = 64;

// Sum of squares over the sixteen lanes of a head.
template <int kSteps> __device__ __forceinline__ float head_squares(const float (&x)[kSteps][8]) {
  float ss = 0.f;
#pragma unroll
  for (int s = 0; s < kSteps; ++s)
#pragma unroll
    for (int i = 0; i < 8; ++i) ss = fmaf(x[s][i], x[s][i], ss);
  return row16_sum(ss);
}

// Sixteen lanes take kUnits heads of one row that turn by the same table (q and k heads, or v heads), so that the row's
// angles are read once for all of them; kSteps steps of 128 dims.  kRow: the workgroup is one row, normed as a whole.
template <typename T, int kSteps, int kUnits, bool kRow>
__global__ __launch_bounds__(kRow ? 16 * kMaxRowParts : 256) void head_rope_store_kernel(const HeadRopeArgs a, unsigned parts_qk, unsigned parts) {
  const unsigned item = kRow ? threadIdx.x / kLanes : blockIdx.x * (256 / kLanes) + threadIdx.x / kLanes;
  const int li = threadIdx.x % kLanes;
  const bool live = item < (kRow ? parts : (unsigned)a.rows * parts);
  const int64_t t = kRow ? (int64_t)blockIdx.x : live ? item / parts : 0;
  const unsigned part = !live ? 0 : kRow ? item : item - (unsigned)t * parts;
  const bool is_v = part >= parts_qk;
  const int u0 = (int)(is_v ? part - parts_qk : part) * kUnits;        // first head: q and k heads counted through, or v heads
  const int count = live ? min(kUnits, (is_v ? a.kv_heads : a.heads + a.kv_heads) - u0) : 0;
  const int n = is_v ? a.vdim : a.dim;
  const T* src = reinterpret_cast<const T*>(a.proj) + t * a.proj_stride + (is_v ? (int64_t)(a.heads + a.kv_heads) * a.dim : 0) + (int64_t)u0 * n;
  float x[kUnits][kSteps][8];
#pragma unroll
  for (int j = 0; j < kUnits; ++j)
#pragma unroll
    for (int s = 0; s < kSteps; ++s) {
      const int d0 = 8 * (li + kLanes * s);
#pragma unroll
      for (int i = 0; i < 8; ++i) x[j][s][i] = 0.f;
      if (j < count && d0 < n) load8(src + j * n + d0, min(8, n - d0), x[j][s]);
    }
  int64_t pos = a.positions[t];
  pos = pos < 0 ? 0 : pos >= a.max_position ? a.max_position - 1 : pos;
  const int rot = is_v ? (a.v_table ? a.vdim : 0) : (a.rot_table ? a.rot : 0);
  const float2* cs = rot == 0 ? nullptr : (is_v ? a.v_table : a.rot_table) + pos * (rot / 2);
  const int64_t dst = a.dst_row ? a.dst_row[t] : t, kv_dst = a.kv_row ? a.kv_row[t] : dst;
  const int64_t own_slot = a.slots ? a.slots[t] : -1;
  float row_scale[2] = {1.f, 1.f};                                     // of q and of k
  if constexpr (kRow) {
    __shared__ float squares[2][kMaxRowParts];
    float mine[2] = {0.f, 0.f};
#pragma unroll
    for (int j = 0; j < kUnits; ++j) {
      const float ss = head_squares(x[j]);                             // heads that are not there are zeros
      if (!is_v) mine[u0 + j >= a.heads] += ss;
    }
    if (li == 0) {
      squares[0][item] = live ? mine[0] : 0.f;
      squares[1][item] = live ? mine[1] : 0.f;
    }
    __syncthreads();
    const unsigned groups = blockDim.x / kLanes;
#pragma unroll
    for (int w = 0; w < 2; ++w) {
      float ss = 0.f;
      for (unsigned i = li; i < groups; i += kLanes) ss += squares[w][i];
      row_scale[w] = 1.0f / sqrtf(row16_sum(ss) / (float)((w == 0 ? a.heads : a.kv_heads) * n) + a.eps);
    }
  }
  float2 angle[kSteps][4];                                             // of the lane's pairs (interleaved layout)
#pragma unroll
  for (int s = 0; s < kSteps; ++s) load_angles(angle[s], cs, 8 * (li + kLanes * s), a.interleaved ? rot : 0);
#pragma unroll
  for (int j = 0; j < kUnits; ++j) {
    const int u = u0 + j;
    const bool is_q = !is_v && u < a.heads;
    const int head = is_q || is_v ? u : u - a.heads;
    const float* gain = is_v ? nullptr : is_q ? a.gain_q : a.gain_k;
    float scale = 1.f;
    if constexpr (kRow) {
      scale = row_scale[is_q ? 0 : 1];
      if (gain && j < count) gain += (int64_t)head * a.dim;
    } else if (gain) {                                                 // the same for the sixteen lanes
      scale = 1.0f / sqrtf(head_squares(x[j]) / (float)n + a.eps);
    }
    // what follows the rotation; a rotation by unequal angles keeps a head's squares only up to the table's amplitude
    const bool unit = is_v ? (a.norms & kNormValues) != 0 : (a.norms & kNormTurned) != 0;
    if (j < count) {
#pragma unroll
      for (int s = 0; s < kSteps; ++s) {
        const int d0 = 8 * (li + kLanes * s);
        if (d0 >= a.D) continue;
        float* v = x[j][s];
        if (gain) {
          float g[8];
          load8(gain + d0, max(min(8, n - d0), 0), g);
#pragma unroll
          for (int i = 0; i < 8; ++i) v[i] = v[i] * scale * g[i];
        }
        if (d0 < rot) {
          if (a.interleaved) {
            turn_pairs(v, angle[s], 1.f);
          } else {
            float partner[8];
            load_partner(src + j * n, gain, scale, d0, rot, partner);
            turn_halves(v, partner, d0, rot, cs, 1.f);
          }
        }
      }
    }
    float factor = unit ? 1.0f / sqrtf(head_squares(x[j]) / (float)n + a.eps) : 1.f;
    if (j >= count) continue;
    if (is_q) factor *= a.head_scale ? a.q_scale * a.head_scale[head] : a.q_scale;
    T* packed = reinterpret_cast<T*>(is_q ? a.q_out : is_v ? a.v_out : a.k_out);
    if (packed && is_q) packed += (dst * a.heads + head) * a.D;
    else if (packed) packed = kv_dst < 0 ? nullptr : packed + (kv_dst * a.kv_heads + head) * a.kv_head;
    const int64_t slot = is_q ? -1 : own_slot;
    T* cached = nullptr;
    if (slot >= 0 && slot < a.num_slots) cached = reinterpret_cast<T*>(is_v ? a.v_cache : a.k_cache) + (slot * a.kv_heads + head) * a.kv_head;
#pragma unroll
    for (int s = 0; s < kSteps; ++s) {
      const int d0 = 8 * (li + kLanes * s);
      if (d0 >= a.D) continue;
      float* v = x[j][s];
      if (is_q || unit) {
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] *= factor;
      }
      const int m = min(8, a.D - d0);
      if (packed) store8(packed + d0, m, v);
      if (cached) store8(cached + d0, m, v);
    }
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

template <typename T, int kSteps, int kUnits>
__global__ __launch_bounds__(256) void head_unrotate_gate_kernel(const UnrotateGateArgs a, unsigned parts) {
  const unsigned item = blockIdx.x * (256 / kLanes) + threadIdx.x / kLanes;
  const int li = threadIdx.x % kLanes;
  if (item >= (unsigned)a.rows * parts) return;
  const int64_t t = item / parts;
  const int h0 = (int)(item - (unsigned)t * parts) * kUnits, count = min(kUnits, a.heads - h0);
  const int64_t src_row = a.dst_row ? a.dst_row[t] : t;
  const T* src = reinterpret_cast<const T*>(a.o) + (src_row * a.heads + h0) * a.D;
  T* dst = reinterpret_cast<T*>(a.out) + (t * a.heads + h0) * a.vdim;
  float x[kUnits][kSteps][8], g[kUnits];
#pragma unroll
  for (int j = 0; j < kUnits; ++j) {
#pragma unroll
    for (int s = 0; s < kSteps; ++s) {
      const int d0 = 8 * (li + kLanes * s);
      if (j < count && d0 < a.vdim) load8(src + j * a.D + d0, min(8, a.vdim - d0), x[j][s]);
    }
    g[j] = 1.f;
    if (a.gate && j < count) g[j] = 1.0f / (1.0f + __expf(-to_float(reinterpret_cast<const T*>(a.gate)[t * a.gate_stride + h0 + j])));
  }
  int64_t pos = a.positions[t];
  pos = pos < 0 ? 0 : pos >= a.max_position ? a.max_position - 1 : pos;
  const int rot = a.v_table ? a.vdim : 0;
  const float2* cs = rot ? a.v_table + pos * (rot / 2) : nullptr;
#pragma unroll
  for (int s = 0; s < kSteps; ++s) {
    const int d0 = 8 * (li + kLanes * s);
    if (d0 >= a.vdim) continue;
    float2 angle[4];
    load_angles(angle, cs, d0, a.interleaved ? rot : 0);
#pragma unroll
    for (int j = 0; j < kUnits; ++j) {
      if (j >= count) break;
      if (d0 < rot) {
        if (a.interleaved) {
          turn_pairs(x[j][s], angle, -1.f);
        } else {
          float partner[8];
          load_partner(src + j * a.D, nullptr, 1.f, d0, rot, partner);
          turn_halves(x[j][s], partner, d0, rot, cs, -1.f);
        }
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) x[j][s][i] *= g[j];
      store8(dst + j * a.vdim + d0, min(8, a.vdim - d0), x[j][s]);
    }
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

constexpr int kRowUnits = 4;       // heads per sixteen lanes where there are rows enough to fill the chip anyway
constexpr int kManyRows = 512;

static unsigned head_blocks(int64_t items) { return (unsigned)((items + 256 / kLanes - 1) / (256 / kLanes)); }

// f(steps, units): compile-time counts of 128-dim steps and of heads per sixteen lanes
template <typename F> static void with_steps(int head_dim, int64_t rows, F f) {
  using std::integral_constant;
  if (head_dim > 8 * kLanes) f(integral_constant<int, kMaxSteps>{}, integral_constant<int, 1>{});
  else if (rows < kManyRows) f(integral_constant<int, 1>{}, integral_constant<int, 1>{});
  else f(integral_constant<int, 1>{}, integral_constant<int, kRowUnits>{});
}

extern "C" int mvllm_head_norm_rope_store(void* q_out, void* k_out, void* v_out, const int64_t* kv_row, const void* proj,
                                          int64_t proj_row_stride, const float* gain_q, const float* gain_k, int norms, float eps,
                                          float q_scale, const float* head_scale, const float* rot_table, int rot_dims,
                                          const float* v_table, int interleaved, int64_t max_position, const int64_t* positions,
                                          const int32_t* dst_row, const int64_t* slots, void* k_cache, void* v_cache,
                                          int kv_head_stride, int64_t num_slots, int64_t rows, int num_heads, int num_kv_heads,
                                          int dim, int vdim, int head_dim, int dtype, void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || num_heads <= 0 || num_kv_heads <= 0 || num_heads % num_kv_heads != 0 || dim <= 0 || vdim <= 0 ||
      head_dim < dim || head_dim < vdim || rot_dims < 0 || rot_dims > dim || rot_dims % 2 != 0 || kv_head_stride < head_dim ||
      (v_table && vdim % 2 != 0) || max_position <= 0 || num_slots < 0 || norms < 0 || norms > 7 ||
      ((norms & kNormRows) && (!gain_q || !gain_k)) || proj_row_stride < (int64_t)num_heads * dim + (int64_t)num_kv_heads * (dim + vdim))
    return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || head_dim > 8 * kLanes * kMaxSteps || rows > ((int64_t)1 << 31) / (num_heads + 2 * (int64_t)num_kv_heads))
    return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0) return MVLLM_OK;
  if (!q_out || !proj || !positions || (slots && (!k_cache || !v_cache)) || (rot_dims && !rot_table)) return MVLLM_ERR_NULL_POINTER;
  HeadRopeArgs a;
  a.q_out = q_out; a.k_out = k_out; a.v_out = v_out; a.proj = proj; a.gain_q = gain_q; a.gain_k = gain_k; a.head_scale = head_scale;
  a.rot_table = rot_dims ? reinterpret_cast<const float2*>(rot_table) : nullptr;
  a.v_table = reinterpret_cast<const float2*>(v_table);
  a.positions = positions; a.dst_row = dst_row; a.kv_row = kv_row; a.slots = slots; a.k_cache = k_cache; a.v_cache = v_cache;
  a.proj_stride = proj_row_stride; a.max_position = max_position; a.num_slots = num_slots; a.rows = rows;
  a.heads = num_heads; a.kv_heads = num_kv_heads; a.dim = dim; a.vdim = vdim; a.D = head_dim; a.rot = rot_dims;
  a.interleaved = interleaved; a.norms = norms; a.kv_head = kv_head_stride; a.eps = eps; a.q_scale = q_scale;
  int st = MVLLM_OK;
  auto launch = [&](auto STEPS, auto UNITS) {
    constexpr int kSteps = decltype(STEPS)::value, kUnits = decltype(UNITS)::value;
    const unsigned parts_qk = (unsigned)(num_heads + num_kv_heads + kUnits - 1) / kUnits, parts = parts_qk + (unsigned)(num_kv_heads + kUnits - 1) / kUnits;
    hipStream_t s = (hipStream_t)stream;
    if (norms & kNormRows) {
      if (parts > (unsigned)kMaxRowParts) {
        st = MVLLM_ERR_UNSUPPORTED;
        return;
      }
      const dim3 grid((unsigned)rows), block((parts * kLanes + 63) / 64 * 64);
      if (dtype == MVLLM_F32) head_rope_store_kernel<float, kSteps, kUnits, true><<<grid, block, 0, s>>>(a, parts_qk, parts);
      else head_rope_store_kernel<bf16_t, kSteps, kUnits, true><<<grid, block, 0, s>>>(a, parts_qk, parts);
    } else {
      const dim3 grid(head_blocks(rows * parts));
      if (dtype == MVLLM_F32) head_rope_store_kernel<float, kSteps, kUnits, false><<<grid, dim3(256), 0, s>>>(a, parts_qk, parts);
      else head_rope_store_kernel<bf16_t, kSteps, kUnits, false><<<grid, dim3(256), 0, s>>>(a, parts_qk, parts);
    }
  };
  // more heads than one per sixteen lanes can take side by side: several each, whatever the number of rows
  const bool wide = (norms & kNormRows) && num_heads + 2 * num_kv_heads > kMaxRowParts;
  with_steps(head_dim, wide ? (int64_t)kManyRows : rows, launch);
  return st != MVLLM_OK ? st : launch_status();
}

extern "C" int mvllm_head_rope_store(void* q_out, void* k_out, void* v_out, const void* proj, int64_t proj_row_stride,
                                     const float* gain_q, const float* gain_k, float eps, float q_scale,
                                     const float* rot_table, int rot_dims, const float* v_table, int interleaved,
                                     int64_t max_position, const int64_t* positions, const int32_t* dst_row,
                                     const int64_t* slots, void* k_cache, void* v_cache, int64_t num_slots, int64_t rows,
                                     int num_heads, int num_kv_heads, int dim, int vdim, int head_dim, int dtype,
                                     void* stream) {
  return mvllm_head_norm_rope_store(q_out, k_out, v_out, nullptr, proj, proj_row_stride, gain_q, gain_k, 0, eps, q_scale, nullptr,
                                    rot_table, rot_dims, v_table, interleaved, max_position, positions, dst_row, slots, k_cache,
                                    v_cache, head_dim, num_slots, rows, num_heads, num_kv_heads, dim, vdim, head_dim, dtype, stream);
}

extern "C" int mvllm_head_unrotate_gate(void* out, const void* o, const void* gate, int64_t gate_row_stride,
                                        const float* v_table, int interleaved, int64_t max_position,
                                        const int64_t* positions, const int32_t* dst_row, int64_t rows, int num_heads,
                                        int vdim, int head_dim, int dtype, void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || num_heads <= 0 || vdim <= 0 || head_dim < vdim || (v_table && vdim % 2 != 0) || max_position <= 0 ||
      (gate && gate_row_stride < num_heads))
    return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || head_dim > 8 * kLanes * kMaxSteps || rows > ((int64_t)1 << 31) / num_heads) return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0) return MVLLM_OK;
  if (!out || !o || !positions) return MVLLM_ERR_NULL_POINTER;
  UnrotateGateArgs a;
  a.out = out; a.o = o; a.gate = gate; a.v_table = reinterpret_cast<const float2*>(v_table); a.positions = positions;
  a.dst_row = dst_row; a.gate_stride = gate_row_stride; a.max_position = max_position; a.rows = rows;
  a.heads = num_heads; a.vdim = vdim; a.D = head_dim; a.interleaved = interleaved;
  with_steps(head_dim, rows, [&](auto STEPS, auto UNITS) {
    constexpr int kSteps = decltype(STEPS)::value, kUnits = decltype(UNITS)::value;
    const unsigned parts = (unsigned)(num_heads + kUnits - 1) / kUnits;
    const dim3 grid(head_blocks(rows * parts));
    if (dtype == MVLLM_F32) head_unrotate_gate_kernel<float, kSteps, kUnits><<<grid, dim3(256), 0, (hipStream_t)stream>>>(a, parts);
    else head_unrotate_gate_kernel<bf16_t, kSteps, kUnits><<<grid, dim3(256), 0, (hipStream_t)stream>>>(a, parts);
  });
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
