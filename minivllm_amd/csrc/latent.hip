// Attention over latents: the cache keeps one row c [rank] per token, and per head k = U_k c, v = U_v c.  Since
//     q . (U_k c) = (U_k^T q) . c        and        sum_j p_j U_v c_j = U_v (sum_j p_j c_j)
// a query row can be answered from the latents alone: q' = U_k^T q per head (head_linear), softmax over q' . c with the
// latents as both keys and values (latent_decode: all heads of a row read a latent once), then U_v per head (head_linear).
// That is the form for decoded tokens and short portions; long portions make keys and values of the latents (a matrix
// product) and run the prefill kernels.
//   latent_norm_store   c = rms(row) * weight, packed and into the cache
//   head_linear         out[t, h] = W_h x[t, h]
//   latent_decode       one query row per (row, block of heads, share of the keys); latent_merge joins the shares
// The rank is padded to a multiple of 32 with zeros; scores, weights and sums are fp32.
#include "prefill_tiles.h"

#pragma clang fp contract(off)

namespace mvllm {

// ---- norm and store ----
struct LatentNormArgs {
  void* out;                // [T, padded] or null
  const void* in;           // [T, in_stride]
  const float* weight;      // [rank]
  void* cache;              // [num_slots, padded] or null
  const int64_t* slots;     // [T], < 0: not stored
  int64_t in_stride, num_slots;
  float eps;
  int rows, rank, padded;
  bool vec;                 // the weight starts on 16 bytes
};

// One row per wave, 16 bytes per lane and access.
template <typename T, int NC>
__global__ __launch_bounds__(256) void latent_norm_kernel(const LatentNormArgs a) {
  constexpr int N = 16 / (int)sizeof(T);
  const int row = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (row >= a.rows) return;
  const T* in = reinterpret_cast<const T*>(a.in) + (int64_t)row * a.in_stride;
  const int64_t slot = a.slots ? a.slots[row] : -1;
  float x[NC][N], w[NC][N], ss = 0.f;
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int at = (c * 64 + lane) * N;
    if (at + N <= a.rank && a.vec) {
#pragma unroll
      for (int i = 0; i < N; i += 4) *reinterpret_cast<float4*>(&w[c][i]) = *reinterpret_cast<const float4*>(a.weight + at + i);
    } else {
#pragma unroll
      for (int i = 0; i < N; ++i) w[c][i] = a.weight[min(at + i, a.rank - 1)];
    }
  }
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
  }
  ss = four_rows_sum(row16_sum(ss));
  const float inv = 1.0f / sqrtf(ss / (float)a.rank + a.eps);
  T* out = a.out ? reinterpret_cast<T*>(a.out) + (int64_t)row * a.padded : nullptr;
  T* cached = a.cache && slot >= 0 && slot < a.num_slots ? reinterpret_cast<T*>(a.cache) + slot * a.padded : nullptr;
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int at = (c * 64 + lane) * N;
    if (at >= a.padded) continue;
    T v[N];
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] = from_float<T>(at + i < a.rank ? x[c][i] * inv * w[c][i] : 0.f);
    const uint4 r = *reinterpret_cast<const uint4*>(v);
    if (out) *reinterpret_cast<uint4*>(out + at) = r;
    if (cached) *reinterpret_cast<uint4*>(cached + at) = r;
  }
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

// ---- attention of single rows over the cache ----
struct LatentDecodeArgs {
  void* out;                 // [rows, H, padded]
  const void* q;             // [rows, H, padded]
  const void* cache;         // [num_blocks, block_size, padded]
  const int32_t* tables;     // [entries, table_width]
  const int32_t* row_entry;  // [rows]
  const int64_t* lens;       // [rows]: keys the row sees
  float* part_o;             // [rows, parts, H, padded] (parts > 1)
  float2* part_ml;           // [rows, parts, H]: maximum (base 2), sum
  int64_t num_blocks;
  int table_width, block_size, heads, padded, parts;
  float scale_log2;
};

// Keys of share `part`: whole tiles of 64, all shares of a row as even as that allows.
__device__ __forceinline__ void key_share(const LatentDecodeArgs& a, int row, int part, int& k0, int& k1) {
  const int64_t most = (int64_t)a.table_width * a.block_size;
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
template <typename T>
__device__ __forceinline__ void store4(const LatentDecodeArgs& a, int row, int part, int h, int col, const float* o, float inv) {
  if (a.parts == 1) {
    T* p = reinterpret_cast<T*>(a.out) + ((int64_t)row * a.heads + h) * a.padded + col;
    T v[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = from_float<T>(o[i] * inv);
    if constexpr (sizeof(T) == 4) *reinterpret_cast<uint4*>(p) = *reinterpret_cast<const uint4*>(v);
    else *reinterpret_cast<uint2*>(p) = *reinterpret_cast<const uint2*>(v);
  } else {
    float* p = a.part_o + (((int64_t)row * a.parts + part) * a.heads + h) * a.padded + col;
    *reinterpret_cast<float4*>(p) = make_float4(o[0], o[1], o[2], o[3]);
  }
}

// bf16: workgroup = (share, block of 16 HT heads, row), four waves; RS = padded rank / 32.  Tiles of 64 latents go to LDS
// once, in chunks of 16 bytes whose place in a row is xor-ed with the key's low bits; wave w takes 16-head tile w % HT and
// the key subtiles of its share w / HT.  S^T = C Q'^T (keys down the accumulator, heads across the lanes), so that the
// weights are the operand of O^T += C^T P^T as they lie; C^T comes from the same LDS tile through the transposing loads.  Two
// tiles in LDS: the next one is on its way while this one is worked on.
template <int RS, int HT>
__global__ __launch_bounds__(256, RS > 8 ? 1 : RS > 4 ? 2 : 3) void latent_decode_kernel(const LatentDecodeArgs a) {
  constexpr int kShares = 4 / HT, kSub = 4 / kShares;      // key shares of a tile, 16-key subtiles of a wave
  constexpr int RC = 4 * RS, kRow = 16 * RC;               // chunks and bytes of a row
  constexpr int kXor = (RC & -RC) < 16 ? (RC & -RC) : 16;  // chunks that trade places
  constexpr int kTile = 64 * kRow;
  __shared__ __attribute__((aligned(16))) char lds[2 * kTile];
  __shared__ int64_t slot_of[2][64];
  __shared__ float2 ml[4][16];
  const int part = blockIdx.x, row = blockIdx.z;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), g = lane >> 4, i16 = lane & 15;
  const int ht = wave % HT, share = wave / HT;
  const int h = (blockIdx.y * HT + ht) * 16 + i16;         // this lane's head (as column)
  int k0, k1;
  key_share(a, row, part, k0, k1);
  const int32_t* table = a.tables + (int64_t)a.row_entry[row] * a.table_width;

  uint4 qf[RS];
  {
    const bf16_t* q = reinterpret_cast<const bf16_t*>(a.q) + ((int64_t)row * a.heads + min(h, a.heads - 1)) * (32 * RS) + 8 * g;
#pragma unroll
    for (int ks = 0; ks < RS; ++ks) qf[ks] = *reinterpret_cast<const uint4*>(q + 32 * ks);
  }
  v4f o[2 * RS];
#pragma unroll
  for (int n = 0; n < 2 * RS; ++n) o[n] = v4f{0.f, 0.f, 0.f, 0.f};
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

  // a tile: RS chunks per thread, straight into LDS
  auto copy = [&](int buffer) __attribute__((always_inline)) {
    const char* cache = reinterpret_cast<const char*>(a.cache);
#pragma unroll
    for (int i = 0; i < RS; ++i) {
      const uint32_t c = 256u * i + (uint32_t)tid;
      const uint32_t key = c / RC, p = c % RC;
      const char* from = cache + slot_of[buffer][key] * kRow + ((p ^ (key & (kXor - 1))) << 4);
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
        s[t][r] = at < k1 ? s[t][r] * a.scale_log2 : -INFINITY;
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
      for (int n = 0; n < 2 * RS; ++n) o[n] *= keep;
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
    for (int n = 0; n < 2 * RS; ++n) {
      auto column = [&](int t) __attribute__((always_inline)) {
        const char* p = col_at[n % kCols] + at_tile + 16 * t * kRow + 32 * (n / kCols * kCols);
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
    float4* box = reinterpret_cast<float4*>(lds) + ht * 2 * RS * 64;
    for (int other = 1; other < kShares; ++other) {
      if (share == other) {
#pragma unroll
        for (int n = 0; n < 2 * RS; ++n) box[n * 64 + lane] = make_float4(o[n][0], o[n][1], o[n][2], o[n][3]);
        if (g == 0) ml[ht][i16] = make_float2(m, l);
      }
      __syncthreads();
      if (share == 0) {
        const float2 x = ml[ht][i16];
        const float m_new = fmaxf(m, x.x);
        const float mine = m == -INFINITY ? 0.f : fast_exp2(m - m_new), theirs = x.x == -INFINITY ? 0.f : fast_exp2(x.x - m_new);
#pragma unroll
        for (int n = 0; n < 2 * RS; ++n) {
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
  if (share != 0 || h >= a.heads) return;
  const float inv = l > 0.f ? 1.0f / l : 0.f;
  if (a.parts > 1 && g == 0) a.part_ml[((int64_t)row * a.parts + part) * a.heads + h] = make_float2(m, l);
  if (a.parts > 1 && m == -INFINITY) return;                // the merge reads nothing of it
#pragma unroll
  for (int n = 0; n < 2 * RS; ++n) {
    const float x[4] = {o[n][0], o[n][1], o[n][2], o[n][3]};
    store4<bf16_t>(a, row, part, h, 16 * n + 4 * g, x, inv);
  }
}

// Any type and rank up to 64 NE: workgroup = (share, head, row); a wave takes every fourth key, its lanes the columns.
template <typename T, int NE>
__global__ __launch_bounds__(256) void latent_decode_any_kernel(const LatentDecodeArgs a) {
  __shared__ float part_o[4][64 * NE];
  __shared__ float2 ml[4];
  const int part = blockIdx.x, h = blockIdx.y, row = blockIdx.z;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  int k0, k1;
  key_share(a, row, part, k0, k1);
  const int32_t* table = a.tables + (int64_t)a.row_entry[row] * a.table_width;
  const T* q_row = reinterpret_cast<const T*>(a.q) + ((int64_t)row * a.heads + h) * a.padded;
  float q[NE], o[NE];
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int c = lane + 64 * i;
    q[i] = c < a.padded ? to_float(q_row[c]) * a.scale_log2 : 0.f;
    o[i] = 0.f;
  }
  float m = -INFINITY, l = 0.f;
  constexpr int kTogether = NE > 8 ? 2 : 4;
  for (int base = k0 + wave * kTogether; base < k1; base += 4 * kTogether) {
    float c[kTogether][NE], s[kTogether];
#pragma unroll
    for (int j = 0; j < kTogether; ++j) {
      const T* p = reinterpret_cast<const T*>(a.cache) + key_slot(a, table, min(base + j, k1 - 1)) * a.padded;
      s[j] = 0.f;
#pragma unroll
      for (int i = 0; i < NE; ++i) {
        c[j][i] = lane + 64 * i < a.padded ? to_float(p[lane + 64 * i]) : 0.f;
        s[j] = fmaf(q[i], c[j][i], s[j]);
      }
    }
    float m_new = m;
#pragma unroll
    for (int j = 0; j < kTogether; ++j) {
      s[j] = base + j < k1 ? wave_sum(s[j]) : -INFINITY;
      m_new = fmaxf(m_new, s[j]);
    }
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
  for (int c = 4 * threadIdx.x; c < a.padded; c += 1024) {
    float x[4];
#pragma unroll
    for (int e = 0; e < 4; ++e)
      x[e] = w[0] * part_o[0][c + e] + w[1] * part_o[1][c + e] + w[2] * part_o[2][c + e] + w[3] * part_o[3][c + e];
    store4<T>(a, row, part, h, c, x, inv);
  }
}

// Joins the shares of a (row, head): one wave each, four columns per lane and step.
template <typename T>
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
  const float l = wave_sum(w * x.y);
  const float f = l > 0.f ? w / l : 0.f;
  for (int c = 4 * lane; c < a.padded; c += 256) {
    float o[4] = {0.f, 0.f, 0.f, 0.f};
    for (int p = 0; p < a.parts; ++p) {
      const float g = __shfl(f, p, 64);
      if (g == 0.f) continue;                       // empty shares have left nothing (uniform over the wave)
      const float4 v = *reinterpret_cast<const float4*>(a.part_o + ((row * a.parts + p) * a.heads + h) * a.padded + c);
      o[0] = fmaf(g, v.x, o[0]); o[1] = fmaf(g, v.y, o[1]); o[2] = fmaf(g, v.z, o[2]); o[3] = fmaf(g, v.w, o[3]);
    }
    T v[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = from_float<T>(o[i]);
    T* out = reinterpret_cast<T*>(a.out) + (row * a.heads + h) * a.padded + c;
    if constexpr (sizeof(T) == 4) *reinterpret_cast<uint4*>(out) = *reinterpret_cast<const uint4*>(v);
    else *reinterpret_cast<uint2*>(out) = *reinterpret_cast<const uint2*>(v);
  }
}

template <int RS>
static int launch_decode(const LatentDecodeArgs& a, int rows, hipStream_t s) {
  const int tiles = (a.heads + 15) / 16;
  const dim3 block(256);
  if (tiles == 1) latent_decode_kernel<RS, 1><<<dim3((unsigned)a.parts, 1, (unsigned)rows), block, 0, s>>>(a);
  else if (tiles == 2) latent_decode_kernel<RS, 2><<<dim3((unsigned)a.parts, 1, (unsigned)rows), block, 0, s>>>(a);
  else latent_decode_kernel<RS, 4><<<dim3((unsigned)a.parts, (unsigned)((tiles + 3) / 4), (unsigned)rows), block, 0, s>>>(a);
  return launch_status();
}

template <typename T>
static int launch_any(const LatentDecodeArgs& a, int rows, hipStream_t s) {
  const dim3 grid((unsigned)a.parts, (unsigned)a.heads, (unsigned)rows), block(256);
  if (a.padded <= 128) latent_decode_any_kernel<T, 2><<<grid, block, 0, s>>>(a);
  else if (a.padded <= 512) latent_decode_any_kernel<T, 8><<<grid, block, 0, s>>>(a);
  else if (a.padded <= 1024) latent_decode_any_kernel<T, 16><<<grid, block, 0, s>>>(a);
  else latent_decode_any_kernel<T, 32><<<grid, block, 0, s>>>(a);
  return launch_status();
}

constexpr int kMaxParts = 32;

// Shares per row: as many as give the shortest schedule, in tiles of 64 keys (two more for a share's start and end, two for the
// pass that joins shares), of whole rounds of the workgroups that run side by side.
static int plan_parts(int rows, int heads, int padded, int64_t max_keys, int dtype) {
  const int head_tiles = (heads + 15) / 16;
  const int64_t groups = (int64_t)rows * (dtype == MVLLM_BF16 ? (head_tiles <= 2 ? 1 : (head_tiles + 3) / 4) : heads);
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
  LatentNormArgs a;
  a.out = out; a.in = in; a.weight = weight; a.cache = cache; a.slots = slots; a.in_stride = in_row_stride;
  a.num_slots = num_slots; a.eps = eps; a.rows = (int)rows; a.rank = rank; a.padded = padded; a.vec = aligned16(weight);
  const dim3 grid((unsigned)((rows + 3) / 4)), block(256);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MVLLM_F32) {
    if (padded <= 512) latent_norm_kernel<float, 2><<<grid, block, 0, s>>>(a);
    else latent_norm_kernel<float, 8><<<grid, block, 0, s>>>(a);
  } else {
    if (padded <= 512) latent_norm_kernel<bf16_t, 1><<<grid, block, 0, s>>>(a);
    else latent_norm_kernel<bf16_t, 4><<<grid, block, 0, s>>>(a);
  }
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
  const int parts = plan_parts(rows, num_heads, padded, max_keys, dtype);
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
  LatentDecodeArgs a;
  a.out = out; a.q = q; a.cache = cache; a.tables = block_tables; a.row_entry = row_entry; a.lens = lens;
  a.num_blocks = num_blocks; a.table_width = table_width; a.block_size = block_size; a.heads = num_heads; a.padded = padded;
  a.scale_log2 = scale * kLog2e;
  a.parts = plan_parts(rows, num_heads, padded, (int64_t)table_width * block_size, dtype);
  a.part_o = nullptr;
  a.part_ml = nullptr;
  if (a.parts > 1) {
    if (!workspace || !aligned16(workspace) || workspace_bytes < mvllm_latent_decode_workspace_bytes(rows, num_heads, padded, (int64_t)table_width * block_size, dtype))
      return MVLLM_ERR_WORKSPACE;
    a.part_o = reinterpret_cast<float*>(workspace);
    a.part_ml = reinterpret_cast<float2*>(a.part_o + (int64_t)rows * a.parts * num_heads * padded);
  }
  hipStream_t s = (hipStream_t)stream;
  int st;
  if (dtype == MVLLM_F32) st = launch_any<float>(a, rows, s);
  else switch (padded) {
    case 32: st = launch_decode<1>(a, rows, s); break;
    case 64: st = launch_decode<2>(a, rows, s); break;
    case 96: st = launch_decode<3>(a, rows, s); break;
    case 128: st = launch_decode<4>(a, rows, s); break;
    case 192: st = launch_decode<6>(a, rows, s); break;
    case 256: st = launch_decode<8>(a, rows, s); break;
    case 384: st = launch_decode<12>(a, rows, s); break;
    case 512: st = launch_decode<16>(a, rows, s); break;
    default: st = launch_any<bf16_t>(a, rows, s);
  }
  if (st != MVLLM_OK || a.parts == 1) return st;
  const dim3 grid((unsigned)(((int64_t)rows * num_heads + 3) / 4)), block(256);
  if (dtype == MVLLM_F32) latent_merge_kernel<float><<<grid, block, 0, s>>>(a, rows);
  else latent_merge_kernel<bf16_t><<<grid, block, 0, s>>>(a, rows);
  return launch_status();
}
