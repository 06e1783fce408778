// Attention of single query rows over a paged cache whose rows are keys and values at once (latents, or keys that are their
// own values), or hold a key and behind it a value: the kernels of latent.hip and window_decode.hip.  The windowed form adds
// kv heads, a ring of places, a distance bias, a query temperature and an output gate.
#pragma once
#include "prefill_tiles.h"

#pragma clang fp contract(off)

namespace mvllm {

struct LatentDecodeArgs {
  void* out;                 // [rows, H, value columns] with strides
  const void* q;             // [rows, H, padded] with strides
  const void* cache;         // [num_blocks, block_size, kv_heads, row]: keys in the first `padded` columns
  const int32_t* tables;     // [entries, table_width]
  const int32_t* row_entry;  // [rows]
  const int64_t* lens;       // [rows]: keys the row sees
  float* part_o;             // [rows, parts, H, value columns] (parts > 1)
  float2* part_ml;           // [rows, parts, H]: maximum (base 2), sum
  int64_t num_blocks;
  int64_t q_row, q_head, out_row, out_head;      // elements
  int table_width, block_size, heads, kv_heads, padded, values, parts;
  int row, value_col;        // columns of a cached row; where its values start (0: they are the keys)
  float scale_log2;
  // the windowed form
  const float* slopes;       // [H] or null: slope * distance is taken off a score (natural units)
  const void* gate;          // [rows, gate_row], head h's columns at h * gate_head (1: one number for all), or null: the result
                             // times sigmoid(gate)
  int64_t gate_row, gate_head;
  int window;                // keys nearer than this are seen; 0: all
  int ring;                  // token p lies at place p mod ring of the table; 0: at place p
  float temp_coef, temp_every;       // scores times 1 + coef ln(floor((p + 1) / every) + 1); every 0: not
  const float* sinks;        // [H] or null (the merge only): one more exp(sink) in a row's denominator
};

// Factor of the scores of a query at position p.
__device__ __forceinline__ float query_temperature(float coef, float every, int64_t p) {
  return every > 0.f ? 1.f + coef * logf((float)floor((double)(p + 1) / (double)every) + 1.f) : 1.f;
}

// How a row of the windowed form sees the places of its table.
template <bool kWindowed> struct RowView {
  int place, ring, window;   // of the row's own token
  float scale_log2;
  __device__ __forceinline__ RowView(const LatentDecodeArgs& a, int row) {
    scale_log2 = a.scale_log2;
    if constexpr (kWindowed) {
      const int64_t p = max(a.lens[row], (int64_t)1) - 1;
      ring = a.ring;
      place = (int)(ring > 0 ? p % ring : p);
      window = a.window > 0 ? a.window : 0x7fffffff;
      scale_log2 *= query_temperature(a.temp_coef, a.temp_every, p);
    }
  }
  // tokens between the row's own and the one at that place (places of later tokens come out as at least the window)
  __device__ __forceinline__ int distance(int at) const {
    const int d = place - at;
    return d < 0 ? d + ring : d;
  }
};

// Keys of share `part`: whole tiles of 64, all shares of a row as even as that allows.
__device__ __forceinline__ void key_share(const LatentDecodeArgs& a, int row, int part, int& k0, int& k1) {
  int64_t most = (int64_t)a.table_width * a.block_size;
  if (a.ring > 0) most = min(most, (int64_t)a.ring);
  const int n = (int)min(max(a.lens[row], (int64_t)0), most);
  const int tiles = (n + 63) / 64, per = (tiles + a.parts - 1) / a.parts;
  k0 = min(part * per * 64, n);
  k1 = min(k0 + per * 64, n);
}

// Cache row of key `at` of the entry.
__device__ __forceinline__ int64_t key_slot(const LatentDecodeArgs& a, const int32_t* table, int at) {
  const int b = at / a.block_size;
  const int64_t block = min(max((int64_t)table[b], (int64_t)0), a.num_blocks - 1);
  return block * a.block_size + (at - b * a.block_size);
}

// Results of a share: the answer itself when there is one share only, otherwise partial sums.
template <typename T, bool kWindowed>
__device__ __forceinline__ void finish4(const LatentDecodeArgs& a, int64_t row, int h, int col, const float* o) {
  T* p = reinterpret_cast<T*>(a.out) + row * a.out_row + h * a.out_head + col;
  T v[4];
  if (kWindowed && a.gate) {
    const bool one = a.gate_head == 1;
    const T* gate = reinterpret_cast<const T*>(a.gate) + row * a.gate_row + h * a.gate_head + (one ? 0 : col);
    T g[4];
    if (one) g[0] = g[1] = g[2] = g[3] = *gate;
    else if constexpr (sizeof(T) == 4) *reinterpret_cast<uint4*>(g) = *reinterpret_cast<const uint4*>(gate);
    else *reinterpret_cast<uint2*>(g) = *reinterpret_cast<const uint2*>(gate);
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = from_float<T>(o[i] / (1.f + expf(-to_float(g[i]))));
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = from_float<T>(o[i]);
  }
  if constexpr (sizeof(T) == 4) *reinterpret_cast<uint4*>(p) = *reinterpret_cast<const uint4*>(v);
  else *reinterpret_cast<uint2*>(p) = *reinterpret_cast<const uint2*>(v);
}

template <typename T, bool kWindowed>
__device__ __forceinline__ void store4(const LatentDecodeArgs& a, int row, int part, int h, int col, const float* o, float inv) {
  if (a.parts == 1) {
    const float x[4] = {o[0] * inv, o[1] * inv, o[2] * inv, o[3] * inv};
    finish4<T, kWindowed>(a, row, h, col, x);
  } else {
    float* p = a.part_o + (((int64_t)row * a.parts + part) * a.heads + h) * a.values + col;
    *reinterpret_cast<float4*>(p) = make_float4(o[0], o[1], o[2], o[3]);
  }
}

// bf16: workgroup = (share, kv head and block of 16 HT of its heads, row), four waves; RS = padded rank / 32, VS = value
// columns / 32 (the first ones of a row, or with SPLIT the ones behind the key).  Tiles of 64 latents go to LDS
// once, in chunks of 16 bytes whose place in a row is xor-ed with the key's low bits; wave w takes 16-head tile w % HT and
// the key subtiles of its share w / HT.  S^T = C Q'^T (keys down the accumulator, heads across the lanes), so that the
// weights are the operand of O^T += C^T P^T as they lie; C^T comes from the same LDS tile through the transposing loads.  Two
// tiles in LDS: the next one is on its way while this one is worked on.
template <int RS, int VS, int HT, bool kWindowed, bool SPLIT = false>
__global__ __launch_bounds__(256, RS + SPLIT * VS > 8 ? 1 : RS + SPLIT * VS > 4 ? 2 : 3) void latent_decode_kernel(const LatentDecodeArgs a) {
  constexpr int kShares = 4 / HT, kSub = 4 / kShares;      // key shares of a tile, 16-key subtiles of a wave
  constexpr int RB = RS + SPLIT * VS, VC = SPLIT ? 2 * RS : 0;     // 32-column blocks of a row; 16-column groups before its values
  constexpr int RC = 4 * RB, kRow = 16 * RC;               // chunks and bytes of a row
  constexpr int kXor = (RC & -RC) < 16 ? (RC & -RC) : 16;  // chunks that trade places
  constexpr int kTile = 64 * kRow;
  __shared__ __attribute__((aligned(16))) char lds[2 * kTile];
  __shared__ int64_t slot_of[2][64];
  __shared__ float2 ml[4][16];
  const int part = blockIdx.x, row = blockIdx.z;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), g = lane >> 4, i16 = lane & 15;
  const int ht = wave % HT, share = wave / HT;
  const int group = kWindowed ? a.heads / a.kv_heads : a.heads, blocks = (group + 16 * HT - 1) / (16 * HT);
  const int kv = kWindowed ? blockIdx.y / blocks : 0;
  const int h_in = ((blockIdx.y - kv * blocks) * HT + ht) * 16 + i16, h = kv * group + h_in;       // this lane's head (as column)
  const int64_t cache_row = (kWindowed ? a.kv_heads : 1) * (int64_t)kRow;
  const RowView<kWindowed> view(a, row);
  float slope = 0.f;
  if (kWindowed && a.slopes) slope = a.slopes[min(h, a.heads - 1)] * kLog2e;
  int k0, k1;
  key_share(a, row, part, k0, k1);
  const int32_t* table = a.tables + (int64_t)a.row_entry[row] * a.table_width;

  uint4 qf[RS];
  {
    const bf16_t* q = reinterpret_cast<const bf16_t*>(a.q) + row * a.q_row + min(h, a.heads - 1) * a.q_head + 8 * g;
#pragma unroll
    for (int ks = 0; ks < RS; ++ks) qf[ks] = *reinterpret_cast<const uint4*>(q + 32 * ks);
  }
  v4f o[2 * VS];
#pragma unroll
  for (int n = 0; n < 2 * VS; ++n) o[n] = v4f{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;

  // places in LDS: only the low bits of a chunk's number depend on the lane
  constexpr int kBy = kXor / 4 > 0 ? kXor / 4 : 1, kCols = kXor / 2;
  const char* key_at[kBy];                         // chunk 4 b + g of key 16 (first subtile) + i16
  const char* col_at[kCols];                       // column group j of key 4 g + i16 / 4 of the first subtile
  {
    const char* row_a = lds + (16 * share * kSub + i16) * kRow;
    const char* row_b = lds + (16 * share * kSub + 4 * g + (i16 >> 2)) * kRow + 8 * (i16 & 1);
    const int xa = i16 & (kXor - 1), xb = (4 * g + (i16 >> 2)) & (kXor - 1);
#pragma unroll
    for (int b = 0; b < kBy; ++b) key_at[b] = row_a + (((4 * b + g) ^ xa) << 4);
#pragma unroll
    for (int j = 0; j < kCols; ++j) col_at[j] = row_b + (((2 * j + ((i16 & 3) >> 1)) ^ xb) << 4);
  }

  // a tile: RB chunks per thread, straight into LDS
  auto copy = [&](int buffer) __attribute__((always_inline)) {
    const char* cache = reinterpret_cast<const char*>(a.cache) + kv * (int64_t)kRow;
#pragma unroll
    for (int i = 0; i < RB; ++i) {
      const uint32_t c = 256u * i + (uint32_t)tid;
      const uint32_t key = c / RC, p = c % RC;
      const char* from = cache + slot_of[buffer][key] * cache_row + ((p ^ (key & (kXor - 1))) << 4);
      dma16_to_lds_from(from, lds_address(lds) + buffer * kTile + (256 * i + 64 * wave) * 16);
      if (i % 4 == 3) __builtin_amdgcn_sched_barrier(0);
    }
  };
  if (tid < 128 && k0 < k1) slot_of[tid >> 6][tid & 63] = key_slot(a, table, min(k0 + tid, k1 - 1));
  __syncthreads();
  if (k0 < k1) copy(0);
  dma_wait_all();
  __syncthreads();
  int flip = 0;
  for (int base = k0; base < k1; base += 64, flip ^= 1) {
    const bool more = base + 64 < k1;
    int64_t slot_after = 0;                         // of the tile behind the next one
    if (tid < 64 && base + 128 < k1) slot_after = key_slot(a, table, min(base + 128 + tid, k1 - 1));
    if (more) copy(flip ^ 1);
    __builtin_amdgcn_sched_barrier(0);
    const int at_tile = flip * kTile;

    // ---- scores of the wave's subtiles ----
    v4f s[kSub];
#pragma unroll
    for (int t = 0; t < kSub; ++t) s[t] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < RS; ++ks) {
#pragma unroll
      for (int t = 0; t < kSub; ++t)
        s[t] = mfma16x16x32<bf16_t>(*reinterpret_cast<const uint4*>(key_at[ks % kBy] + at_tile + 16 * t * kRow + 64 * (ks / kBy * kBy)), qf[ks], s[t]);
      if (ks % 4 == 3) __builtin_amdgcn_sched_barrier(0);      // operands of later steps stay in LDS until then
    }
    float most = -INFINITY;
#pragma unroll
    for (int t = 0; t < kSub; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int at = base + 16 * (share * kSub + t) + 4 * g + r;
        if constexpr (kWindowed) {
          const int d = view.distance(at);
          s[t][r] = at < k1 && d < view.window ? s[t][r] * view.scale_log2 - slope * (float)d : -INFINITY;
        } else {
          s[t][r] = at < k1 ? s[t][r] * view.scale_log2 : -INFINITY;
        }
        most = fmaxf(most, s[t][r]);
      }
    most = fmaxf(most, __shfl_xor(most, 16, 64));
    most = fmaxf(most, __shfl_xor(most, 32, 64));
    // the running maximum moves only when it grows by more than 2^8 (or from nothing): weights stay below that
    if (__any(most > m + 8.f || (m == -INFINITY && most > -INFINITY))) {
      const float m_new = fmaxf(m, most);
      const float keep = m == -INFINITY ? 0.f : fast_exp2(m - m_new);
      m = m_new;
      l *= keep;
#pragma unroll
      for (int n = 0; n < 2 * VS; ++n) o[n] *= keep;
    }
    uint2 w[kSub];
#pragma unroll
    for (int t = 0; t < kSub; ++t) {
      float p[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        p[r] = m == -INFINITY ? 0.f : fast_exp2(s[t][r] - m);
        l += p[r];
      }
      w[t] = make_uint2(pack2<bf16_t>(p[0], p[1]), pack2<bf16_t>(p[2], p[3]));
    }
    // ---- O^T += C^T P^T: 16 columns of the latents at a time ----
#pragma unroll
    for (int n = 0; n < 2 * VS; ++n) {
      auto column = [&](int t) __attribute__((always_inline)) {
        const char* p = col_at[(n + VC) % kCols] + at_tile + 16 * t * kRow + 32 * ((n + VC) / kCols * kCols);
        return __builtin_bit_cast(uint2, __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) v4s*)p));
      };
      if constexpr (kSub == 1) {
        o[n] = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(__builtin_bit_cast(v4s, column(0)), __builtin_bit_cast(v4s, w[0]), o[n], 0, 0, 0);
      } else {
#pragma unroll
        for (int t = 0; t < kSub; t += 2) {
          const uint2 c0 = column(t), c1 = column(t + 1);
          o[n] = mfma16x16x32<bf16_t>(make_uint4(c0.x, c0.y, c1.x, c1.y), make_uint4(w[t].x, w[t].y, w[t + 1].x, w[t + 1].y), o[n]);
        }
      }
      if (n % 4 == 3) __builtin_amdgcn_sched_barrier(0);
    }
    __builtin_amdgcn_sched_barrier(0);
    if (tid < 64 && base + 128 < k1) slot_of[flip][tid] = slot_after;
    dma_wait_all();
    __syncthreads();                                // everybody is done with the tile; the next one and its successor's slots are there
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);

  // ---- the shares of a head tile meet in LDS, one after the other ----
  if constexpr (kShares > 1) {
    float4* box = reinterpret_cast<float4*>(lds) + ht * 2 * VS * 64;
    for (int other = 1; other < kShares; ++other) {
      if (share == other) {
#pragma unroll
        for (int n = 0; n < 2 * VS; ++n) box[n * 64 + lane] = make_float4(o[n][0], o[n][1], o[n][2], o[n][3]);
        if (g == 0) ml[ht][i16] = make_float2(m, l);
      }
      __syncthreads();
      if (share == 0) {
        const float2 x = ml[ht][i16];
        const float m_new = fmaxf(m, x.x);
        const float mine = m == -INFINITY ? 0.f : fast_exp2(m - m_new), theirs = x.x == -INFINITY ? 0.f : fast_exp2(x.x - m_new);
#pragma unroll
        for (int n = 0; n < 2 * VS; ++n) {
          const float4 b = box[n * 64 + lane];
          o[n] = v4f{o[n][0] * mine + b.x * theirs, o[n][1] * mine + b.y * theirs, o[n][2] * mine + b.z * theirs, o[n][3] * mine + b.w * theirs};
          if (n % 4 == 3) __builtin_amdgcn_sched_barrier(0);
        }
        l = l * mine + x.y * theirs;
        m = m_new;
      }
      __syncthreads();
    }
  }
  if (share != 0 || h_in >= group) return;
  const float inv = l > 0.f ? 1.0f / l : 0.f;
  if (a.parts > 1 && g == 0) a.part_ml[((int64_t)row * a.parts + part) * a.heads + h] = make_float2(m, l);
  if (a.parts > 1 && m == -INFINITY) return;                // the merge reads nothing of it
#pragma unroll
  for (int n = 0; n < 2 * VS; ++n) {
    const float x[4] = {o[n][0], o[n][1], o[n][2], o[n][3]};
    store4<bf16_t, kWindowed>(a, row, part, h, 16 * n + 4 * g, x, inv);
  }
}

// Any type and rank up to 64 NE: workgroup = (share, head, row); a wave takes every fourth key, its lanes the columns.
template <typename T, int NE, bool kWindowed>
__global__ __launch_bounds__(256) void latent_decode_any_kernel(const LatentDecodeArgs a) {
  __shared__ float part_o[4][64 * NE];
  __shared__ float2 ml[4];
  const int part = blockIdx.x, h = blockIdx.y, row = blockIdx.z;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  int k0, k1;
  key_share(a, row, part, k0, k1);
  const int32_t* table = a.tables + (int64_t)a.row_entry[row] * a.table_width;
  const T* q_row = reinterpret_cast<const T*>(a.q) + row * a.q_row + h * a.q_head;
  const int kv_heads = kWindowed ? a.kv_heads : 1, kv = kWindowed ? h / (a.heads / a.kv_heads) : 0;
  const RowView<kWindowed> view(a, row);
  const float slope = kWindowed && a.slopes ? a.slopes[h] * kLog2e : 0.f;
  float q[NE], o[NE];
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int c = lane + 64 * i;
    q[i] = c < a.padded ? to_float(q_row[c]) * view.scale_log2 : 0.f;
    o[i] = 0.f;
  }
  float m = -INFINITY, l = 0.f;
  constexpr int kTogether = NE > 8 ? 2 : 4;
  for (int base = k0 + wave * kTogether; base < k1; base += 4 * kTogether) {
    float c[kTogether][NE], s[kTogether];
    const T* from[kTogether];
#pragma unroll
    for (int j = 0; j < kTogether; ++j) {
      const T* p = from[j] = reinterpret_cast<const T*>(a.cache) + (key_slot(a, table, min(base + j, k1 - 1)) * kv_heads + kv) * a.row;
      s[j] = 0.f;
#pragma unroll
      for (int i = 0; i < NE; ++i) {
        c[j][i] = lane + 64 * i < a.padded ? to_float(p[lane + 64 * i]) : 0.f;
        s[j] = fmaf(q[i], c[j][i], s[j]);
      }
    }
    if (kWindowed && a.value_col > 0) {             // the values behind the keys take their place
#pragma unroll
      for (int j = 0; j < kTogether; ++j)
#pragma unroll
        for (int i = 0; i < NE; ++i) c[j][i] = lane + 64 * i < a.values ? to_float(from[j][a.value_col + lane + 64 * i]) : 0.f;
    }
    float m_new = m;
#pragma unroll
    for (int j = 0; j < kTogether; ++j) {
      s[j] = base + j < k1 ? wave_sum(s[j]) : -INFINITY;
      if constexpr (kWindowed) {
        const int d = view.distance(base + j);
        s[j] = d < view.window ? s[j] - slope * (float)d : -INFINITY;
      }
      m_new = fmaxf(m_new, s[j]);
    }
    if (kWindowed && m_new == -INFINITY) continue;  // nothing seen so far
    const float keep = exp2f(m - m_new);            // from nothing: exp2(-inf) = 0
    m = m_new;
    l *= keep;
#pragma unroll
    for (int i = 0; i < NE; ++i) o[i] *= keep;
#pragma unroll
    for (int j = 0; j < kTogether; ++j) {
      const float p = exp2f(s[j] - m);
      l += p;
#pragma unroll
      for (int i = 0; i < NE; ++i) o[i] = fmaf(p, c[j][i], o[i]);
    }
  }
#pragma unroll
  for (int i = 0; i < NE; ++i) part_o[wave][lane + 64 * i] = o[i];
  if (lane == 0) ml[wave] = make_float2(m, l);
  __syncthreads();
  float m_all = -INFINITY, l_all = 0.f, w[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) m_all = fmaxf(m_all, ml[i].x);
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    w[i] = ml[i].x == -INFINITY ? 0.f : exp2f(ml[i].x - m_all);
    l_all = fmaf(w[i], ml[i].y, l_all);
  }
  const float inv = l_all > 0.f ? 1.0f / l_all : 0.f;
  if (a.parts > 1 && threadIdx.x == 0) a.part_ml[((int64_t)row * a.parts + part) * a.heads + h] = make_float2(m_all, l_all);
  for (int c = 4 * threadIdx.x; c < a.values; c += 1024) {
    float x[4];
#pragma unroll
    for (int e = 0; e < 4; ++e)
      x[e] = w[0] * part_o[0][c + e] + w[1] * part_o[1][c + e] + w[2] * part_o[2][c + e] + w[3] * part_o[3][c + e];
    store4<T, kWindowed>(a, row, part, h, c, x, inv);
  }
}

// Joins the shares of a (row, head): one wave each, four columns per lane and step.
template <typename T, bool kWindowed>
__global__ __launch_bounds__(256) void latent_merge_kernel(const LatentDecodeArgs a, int rows) {
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  if (item >= (int64_t)rows * a.heads) return;
  const int64_t row = item / a.heads;
  const int h = (int)(item - row * a.heads);
  // lane p has the maximum and sum of share p (at most 64 shares)
  float2 x = make_float2(-INFINITY, 0.f);
  if (lane < a.parts) x = a.part_ml[(row * a.parts + lane) * a.heads + h];
  const float m = wave_max(x.x);
  const float w = x.x == -INFINITY ? 0.f : exp2f(x.x - m);
  float l = wave_sum(w * x.y);
  if (a.sinks) l = add_sink(l, m, a.sinks[h]);
  const float f = l > 0.f ? w / l : 0.f;
  for (int c0 = 0; c0 < a.values; c0 += 256) {      // every lane goes round as often: the shares' factors come from all of them
    const int c = c0 + 4 * lane;
    const bool mine = c < a.values;
    float o[4] = {0.f, 0.f, 0.f, 0.f};
    for (int p = 0; p < a.parts; ++p) {
      const float g = __shfl(f, p, 64);
      if (g == 0.f) continue;                       // empty shares have left nothing (uniform over the wave)
      const float4 v = *reinterpret_cast<const float4*>(a.part_o + ((row * a.parts + p) * a.heads + h) * a.values + (mine ? c : 0));
      o[0] = fmaf(g, v.x, o[0]); o[1] = fmaf(g, v.y, o[1]); o[2] = fmaf(g, v.z, o[2]); o[3] = fmaf(g, v.w, o[3]);
    }
    if (mine) finish4<T, kWindowed>(a, row, h, c, o);
  }
}

template <int RS, int VS, bool kWindowed, bool SPLIT = false>
static int launch_decode_as(const LatentDecodeArgs& a, int rows, hipStream_t s) {
  const int tiles = (a.heads / a.kv_heads + 15) / 16;
  const dim3 block(256);
  auto grid = [&](int per) { return dim3((unsigned)a.parts, (unsigned)(a.kv_heads * ((tiles + per - 1) / per)), (unsigned)rows); };
  if (tiles == 1) latent_decode_kernel<RS, VS, 1, kWindowed, SPLIT><<<grid(1), block, 0, s>>>(a);
  else if (tiles == 2) latent_decode_kernel<RS, VS, 2, kWindowed, SPLIT><<<grid(2), block, 0, s>>>(a);
  else latent_decode_kernel<RS, VS, 4, kWindowed, SPLIT><<<grid(4), block, 0, s>>>(a);
  return launch_status();
}

template <typename T, bool kWindowed>
static int launch_any(const LatentDecodeArgs& a, int rows, hipStream_t s) {
  const dim3 grid((unsigned)a.parts, (unsigned)a.heads, (unsigned)rows), block(256);
  const int widest = max(a.padded, a.values);
  if (widest <= 128) latent_decode_any_kernel<T, 2, kWindowed><<<grid, block, 0, s>>>(a);
  else if (widest <= 512) latent_decode_any_kernel<T, 8, kWindowed><<<grid, block, 0, s>>>(a);
  else if (widest <= 1024) latent_decode_any_kernel<T, 16, kWindowed><<<grid, block, 0, s>>>(a);
  else latent_decode_any_kernel<T, 32, kWindowed><<<grid, block, 0, s>>>(a);
  return launch_status();
}

// Rows of a key and a value of the same width (window_decode_split.hip), or kNotBuilt.
constexpr int kNotBuilt = 1 << 30;
int launch_decode_split(const LatentDecodeArgs& a, int rows, hipStream_t s);

// Width 576 may be 512 value columns and 64 that only the scores read; every other width is read as values whole.
template <bool kWindowed>
static int launch_decode(const LatentDecodeArgs& a, int rows, int dtype, hipStream_t s) {
  int st = kNotBuilt;
  if (dtype == MVLLM_F32) st = launch_any<float, kWindowed>(a, rows, s);
  else if (a.value_col > 0) {
    if constexpr (kWindowed) st = launch_decode_split(a, rows, s);
    if (st == kNotBuilt) st = launch_any<bf16_t, kWindowed>(a, rows, s);
  } else switch (a.padded) {
    case 32: st = launch_decode_as<1, 1, kWindowed>(a, rows, s); break;
    case 64: st = launch_decode_as<2, 2, kWindowed>(a, rows, s); break;
    case 96: st = launch_decode_as<3, 3, kWindowed>(a, rows, s); break;
    case 128: st = launch_decode_as<4, 4, kWindowed>(a, rows, s); break;
    case 192: st = launch_decode_as<6, 6, kWindowed>(a, rows, s); break;
    case 256: st = launch_decode_as<8, 8, kWindowed>(a, rows, s); break;
    case 384: st = launch_decode_as<12, 12, kWindowed>(a, rows, s); break;
    case 512: st = launch_decode_as<16, 16, kWindowed>(a, rows, s); break;
    case 576:
      if (kWindowed && a.values == 512) {
        st = launch_decode_as<18, 16, true>(a, rows, s);
        break;
      }
      [[fallthrough]];
    default: st = launch_any<bf16_t, kWindowed>(a, rows, s);
  }
  if (st != MVLLM_OK || a.parts == 1) return st;
  const dim3 grid((unsigned)(((int64_t)rows * a.heads + 3) / 4)), block(256);
  if (dtype == MVLLM_F32) latent_merge_kernel<float, kWindowed><<<grid, block, 0, s>>>(a, rows);
  else latent_merge_kernel<bf16_t, kWindowed><<<grid, block, 0, s>>>(a, rows);
  return launch_status();
}

constexpr int kMaxParts = 32;

// Shares per row: as many as give the shortest schedule, in tiles of 64 keys (two more for a share's start and end, two for the
// pass that joins shares), of whole rounds of the workgroups that run side by side.
static int plan_parts(int rows, int heads, int kv_heads, int padded, int64_t max_keys, int dtype) {
  const int head_tiles = (heads / kv_heads + 15) / 16;
  const int64_t groups = (int64_t)rows * (dtype == MVLLM_BF16 ? kv_heads * (head_tiles <= 2 ? 1 : (head_tiles + 3) / 4) : heads);
  const int64_t together = 256 * (dtype != MVLLM_BF16 || padded <= 128 ? 3 : padded <= 256 ? 2 : 1), tiles = (max_keys + 63) / 64;
  int best = 1;
  int64_t best_time = INT64_MAX;
  for (int parts = 1; parts <= kMaxParts && (parts == 1 || 2 * parts <= tiles); ++parts) {
    const int64_t time = (groups * parts + together - 1) / together * ((tiles + parts - 1) / parts + 2) + (parts > 1 ? 2 : 0);
    if (time < best_time) {
      best = parts;
      best_time = time;
    }
  }
  return best;
}

}  // namespace mvllm
