// Windowed attention of long portions (window_prefill.hip, window_prefill_latent.hip): packed queries over packed keys, where an
// entry's keys are its own tokens behind the last ones of its past (cu_k - cu_q tokens more than queries), so that neither a
// ring's places nor what a portion overwrites matter here.  Query i of an entry stands at key (keys - queries) + i and sees the
// `window` keys up to it.
//     score = scale * temperature(p) * (q . [k | k2]) - slope_h * distance,     out = softmax . v  (times sigmoid(gate))
// k2 is a second part of the keys that all heads share (null: none), v null: the values are the keys.  Everything is read where
// the projections left it: row strides, per-head offsets.
//
// bf16 (tiles): workgroup = 4 waves = one kv head x HPW of its query heads x 32-row query tiles; 64-key tiles in LDS, two
// buffers, filled by copies that run during the other one's products; Sᵀ = K Qᵀ, Oᵀ += Vᵀ Pᵀ on v_mfma_f32_32x32x16_bf16, one
// query row per lane (as in prefill_mfma.h).  Values that are the keys are read from the keys' tile.  The first product has one
// more 16-dim step, whose operands are made in registers: against ones on the keys' side the row's negated running maximum as a
// sum of three bf16 numbers (scores leave the matrix unit as exp2 arguments, and the accumulators start from nothing), and for
// the distance bias, against a key's place in its tile and the tile's distance (small integers, exact), the slope in the same
// way; what is constant for a row drops out of the softmax.
#pragma once
#include "prefill_mfma.h"

#pragma clang fp contract(off)

namespace mvllm {

struct WindowPrefillArgs {
  void* out;                  // [total_q, out_row], head h at h * out_head
  const void* q;              // [total_q, q_row], head h at h * q_head: [dim | rot]
  const void* k;              // [total_k, k_row], kv head g at g * k_head: [dim]
  const void* k2;             // [total_k, k2_row]: [rot] or null
  const void* v;              // [total_k, v_row], kv head g at g * v_head: [dim], or null: the keys
  const void* gate;           // [total_q, gate_row], head h at h * gate_head (1: one number for all its columns), or null
  const int32_t* cu_q;        // [num_seqs + 1]
  const int32_t* cu_k;        // [num_seqs + 1]
  const int64_t* positions;   // [total_q] (temperature)
  const float* slopes;        // [heads] or null
  int64_t out_row, out_head, q_row, q_head, k_row, k_head, k2_row, v_row, v_head, gate_row, gate_head;
  int64_t total_q;
  int num_seqs, heads, kv_heads, dim, rot, window, hpw, tiles_x, heads_y, band_bits, band_shift;
  float scale_log2, temp_coef, temp_every;
};

__device__ __forceinline__ float prefill_temperature(const WindowPrefillArgs& a, int64_t row) {
  if (!(a.temp_every > 0.f)) return 1.f;
  return 1.f + a.temp_coef * logf((float)floor((double)(a.positions[row] + 1) / (double)a.temp_every) + 1.f);
}

// Which of a row's 16-byte chunks trade places (xor on the chunk's number), for rows of RC chunks.  Three uses: keys are read
// 16 rows at a time with one chunk, values by the transposing loads as 4 rows x 64 bytes; both have to spread over the banks.
template <int RC> struct Chunks {
  static constexpr int kBits = RC % 16 == 0 ? 16 : RC % 8 == 0 ? 8 : 4;      // places that trade
  static constexpr int kLines = RC % 16 == 0 ? 1 : RC % 8 == 0 ? 2 : 4;      // rows per 256 bytes of banks
  static __device__ __forceinline__ int keys(int row) { return (row / kLines) & (kBits - 1); }
  static __device__ __forceinline__ int values(int row) {
    return kBits == 16 ? ((row & 3) << 2) | (row & 1) : kBits == 8 ? ((row >> 1) & 1) << 2 : 0;
  }
  // both at once; eight rows further down the place changes by xor 2
  static __device__ __forceinline__ int both(int row) {
    const int t = (row / kLines) & (kBits - 1);
    return kBits == 16 ? ((t & 3) << 2) | (t >> 2) : kBits == 8 ? ((t & 1) << 2) | (t >> 1) : t;
  }
};

constexpr int kWinKeys = 64;       // keys per tile

// Copies of a part of a tile, a quarter per wave, 1 KB per instruction.  Where rows divide an instruction the four waves take
// turns, so that a lane's place in a row repeats every sixteen rows: copy i starts from offset i % kStarts and goes on by whole
// rows, which is one number for all lanes.
template <int RC> struct Copies {
  static constexpr int kCount = RC / 4;
  static constexpr bool kEven = 64 % RC == 0;
  static constexpr int kRows = kEven ? 256 / RC : 0;                          // rows the four waves copy at once
  static constexpr int kStarts = !kEven ? kCount : kRows >= 16 ? 1 : 16 / kRows;
  static __device__ __forceinline__ int chunk(int i, int wave, int lane) { return (kEven ? 4 * i + wave : wave * kCount + i) * 64 + lane; }
  static constexpr int lds(int i) { return (kEven ? 4 * i : i) * 1024; }      // behind the wave's first
  static constexpr int kWave = (kEven ? 1 : kCount) * 1024;
};
constexpr int kWinRows = 32;       // query rows per wave

// KS1, KS2: 16-dim steps of the two parts of the keys; TD: 32-dim blocks of the values; SHARED: values are the keys (the form
// with a distance bias).
template <int KS1, int KS2, int TD, bool SHARED>
__global__ __launch_bounds__(256, KS1 > 8 ? 1 : 2) void window_prefill_kernel(const WindowPrefillArgs a) {
  static_assert(KS1 == 2 * TD && (!SHARED || KS2 == 0), "values as wide as the first part of the keys");
  constexpr int RC1 = 2 * KS1, RC2 = KS2 > 0 ? 2 * KS2 : 4, RCV = 4 * TD;
  constexpr int kRow1 = 16 * RC1, kRow2 = 16 * RC2, kRowV = 16 * RCV;
  constexpr int kTile1 = kWinKeys * kRow1, kTile2 = KS2 > 0 ? kWinKeys * kRow2 : 0, kTileV = SHARED ? 0 : kWinKeys * kRowV;
  constexpr int kBuffer = kTile1 + kTile2 + kTileV;
  __shared__ __attribute__((aligned(1024))) char lds[2 * kBuffer];
  auto swz1 = [](int row) __attribute__((always_inline)) { return SHARED ? Chunks<RC1>::both(row) : Chunks<RC1>::keys(row); };
  auto swzv = [](int row) __attribute__((always_inline)) { return SHARED ? Chunks<RCV>::both(row) : Chunks<RCV>::values(row); };

  // ---- work item: (head slice, query tile), dealt as in prefill_mfma.h ----
  const unsigned id = blockIdx.x, slot = id >> 3, xcd = id & 7, round = slot / kXcdChunk;
  const unsigned item = (round * 8 + ((xcd + round) & 7)) * kXcdChunk + slot % kXcdChunk;
  const int BM = kWinRows * (4 / a.hpw);
  int seq_start, seq_len, row0, seq, item_y;
  if (a.num_seqs <= 64) {
    const bool found = a.hpw == 4 ? locate_banded<kWinRows>(a.cu_q, a.num_seqs, item, a.heads_y, a.band_bits, a.band_shift, seq_start, seq_len, row0, seq, item_y)
                     : a.hpw == 2 ? locate_banded<2 * kWinRows>(a.cu_q, a.num_seqs, item, a.heads_y, a.band_bits, a.band_shift, seq_start, seq_len, row0, seq, item_y)
                                  : locate_banded<4 * kWinRows>(a.cu_q, a.num_seqs, item, a.heads_y, a.band_bits, a.band_shift, seq_start, seq_len, row0, seq, item_y);
    if (!found) return;
  } else {
    if (item >= (unsigned)a.tiles_x * (unsigned)a.heads_y) return;
    item_y = (int)(item / (unsigned)a.tiles_x);
    if (!locate_tile(a.cu_q, a.num_seqs, a.tiles_x - 1 - (int)(item % (unsigned)a.tiles_x), BM, seq_start, seq_len, row0, seq)) return;
  }
  item_y = __builtin_amdgcn_readfirstlane(item_y);
  seq_start = __builtin_amdgcn_readfirstlane(seq_start);
  seq_len = __builtin_amdgcn_readfirstlane(seq_len);
  row0 = __builtin_amdgcn_readfirstlane(row0);
  seq = __builtin_amdgcn_readfirstlane(seq);
  const int k_start = a.cu_k[seq], kv_len = a.cu_k[seq + 1] - k_start, cached = kv_len - seq_len;

  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), l32 = lane & 31, hi = lane >> 5;
  const int group = a.heads / a.kv_heads, slices = group / a.hpw;
  const int g = item_y / slices;                                                 // kv head
  const int h = g * group + (item_y % slices) * a.hpw + wave % a.hpw;            // this wave's query head
  const int r0 = row0 + kWinRows * (wave / a.hpw);                               // its first query row
  const bool active = r0 < seq_len;
  const int pos0 = cached + r0;                                                  // that row's key
  const int W = a.window > 0 ? a.window : 0x3fffffff;
  const int j_first = max(0, pos0 - W + 1) / kWinKeys, j_last = min(pos0 + kWinRows - 1, kv_len - 1) / kWinKeys;
  const int wg_first = max(0, cached + row0 - W + 1) / kWinKeys, wg_last = (cached + min(row0 + BM, seq_len) - 1) / kWinKeys;

  // ---- copies ----
  using C1 = Copies<RC1>;
  using C2 = Copies<RC2>;
  using CV = Copies<RCV>;
  constexpr int n1 = C1::kCount, n2 = KS2 > 0 ? C2::kCount : 0, nv = SHARED ? 0 : CV::kCount;
  uint32_t off1[C1::kStarts], off2[C2::kStarts], offv[CV::kStarts];
  const uint32_t row1 = (uint32_t)(a.k_row * 2), row2 = (uint32_t)(a.k2_row * 2), rowv = (uint32_t)(a.v_row * 2);
#pragma unroll
  for (int i = 0; i < C1::kStarts; ++i) {
    const int c = C1::chunk(i, wave, lane), row = c / RC1;
    off1[i] = (uint32_t)row * row1 + (uint32_t)(((c % RC1) ^ swz1(row)) << 4);
  }
#pragma unroll
  for (int i = 0; i < C2::kStarts; ++i) {
    const int c = C2::chunk(i, wave, lane), row = c / RC2;
    off2[i] = (uint32_t)row * row2 + (uint32_t)(((c % RC2) ^ Chunks<RC2>::keys(row)) << 4);
  }
#pragma unroll
  for (int i = 0; i < CV::kStarts; ++i) {
    const int c = CV::chunk(i, wave, lane), row = c / RCV;
    offv[i] = (uint32_t)row * rowv + (uint32_t)(((c % RCV) ^ swzv(row)) << 4);
  }
  const char* k_base = reinterpret_cast<const char*>(a.k) + ((int64_t)k_start * a.k_row + (int64_t)g * a.k_head) * 2;
  const char* k2_base = reinterpret_cast<const char*>(a.k2) + (int64_t)k_start * a.k2_row * 2;
  const char* v_base = reinterpret_cast<const char*>(a.v) + ((int64_t)k_start * a.v_row + (int64_t)g * a.v_head) * 2;
  struct Source { v4i k, k2, v; };
  // Rows past the entry's last key arrive as zeros; nothing is read where `enable` is false.
  auto source = [&](int j, bool enable) __attribute__((always_inline)) {
    const int rows = enable ? min(kv_len - j * kWinKeys, kWinKeys) : 0;
    auto part = [&](const char* base, uint32_t row_bytes, int own) __attribute__((always_inline)) {
      return make_rsrc(base + (int64_t)j * kWinKeys * row_bytes, rows > 0 ? (uint32_t)(rows - 1) * row_bytes + (uint32_t)own : 0u);
    };
    Source s;
    s.k = part(k_base, row1, kRow1);
    s.k2 = KS2 > 0 ? part(k2_base, row2, kRow2) : s.k;
    s.v = SHARED ? s.k : part(v_base, rowv, kRowV);
    return s;
  };
  const uint32_t lds_base = lds_address(lds);
  auto copy = [&](const Source& s, auto C, int buffer) __attribute__((always_inline)) {
    constexpr int c = decltype(C)::value;
    const uint32_t base = lds_base + (uint32_t)(buffer * kBuffer);
    auto go = [&](auto PART, auto I, auto REGION, v4i rsrc, const uint32_t* off, uint32_t row_bytes) __attribute__((always_inline)) {
      using P = decltype(PART);
      constexpr int i = decltype(I)::value, behind = P::kEven ? i / P::kStarts * P::kStarts * P::kRows : 0;       // rows behind the start
      dma16_to_lds_at<decltype(REGION)::value + P::lds(i)>(rsrc, off[i % P::kStarts], (uint32_t)behind * row_bytes, base + (uint32_t)(wave * P::kWave));
    };
    using std::integral_constant;
    if constexpr (c < n1) go(C1{}, integral_constant<int, c>{}, integral_constant<int, 0>{}, s.k, off1, row1);
    else if constexpr (c < n1 + n2) go(C2{}, integral_constant<int, c - n1>{}, integral_constant<int, kTile1>{}, s.k2, off2, row2);
    else go(CV{}, integral_constant<int, c - n1 - n2>{}, integral_constant<int, kTile1 + kTile2>{}, s.v, offv, rowv);
  };
  constexpr int kCopies = n1 + n2 + nv;
  {
    const Source s = source(wg_first, true);
    static_for<kCopies>([&](auto C) { copy(s, C, 0); });
  }

  // ---- queries: column = row l32, dims 16 ks + 8 hi .., times scale, temperature and log2 e ----
  uint4 qf[KS1 + KS2];
  {
    const int64_t row = min((int64_t)seq_start + r0 + l32, a.total_q - 1);
    const bf16_t* src = reinterpret_cast<const bf16_t*>(a.q) + row * a.q_row + (int64_t)h * a.q_head + 8 * hi;
#pragma unroll
    for (int ks = 0; ks < KS1 + KS2; ++ks) qf[ks] = *reinterpret_cast<const uint4*>(src + 16 * ks);
    const float scale = a.scale_log2 * prefill_temperature(a, row);
#pragma unroll
    for (int ks = 0; ks < KS1 + KS2; ++ks) {
      qf[ks].x = scale_pair<bf16_t>(qf[ks].x, scale);
      qf[ks].y = scale_pair<bf16_t>(qf[ks].y, scale);
      qf[ks].z = scale_pair<bf16_t>(qf[ks].z, scale);
      qf[ks].w = scale_pair<bf16_t>(qf[ks].w, scale);
    }
  }
#pragma unroll
  for (int ks = 0; ks < KS1 + KS2; ++ks) asm volatile("" ::"v"(qf[ks].x), "v"(qf[ks].w));   // retired before the copies are counted
  // the further step: lanes of the first half hold the slope times (place in the tile - 64 * tiles up to the wave's last one),
  // the others the running maximum
  uint4 q_more = make_uint4(0u, 0u, 0u, 0u);
  if constexpr (SHARED) {
    const float s = a.slopes ? a.slopes[h] * kLog2e : 0.f;
    const float s0 = to_float(from_float<bf16_t>(s)), s1 = to_float(from_float<bf16_t>(s - s0)), s2 = s - s0 - s1;
    if (hi == 0)
      q_more = make_uint4(pack2<bf16_t>(s0, s1), pack2<bf16_t>(s2, -64.f * s0), pack2<bf16_t>(-64.f * s1, -64.f * s2),
                          pack2<bf16_t>(-16384.f * s0, -16384.f * s1));
  }
  const uint32_t ones = hi ? 0x3f803f80u : 0u;       // keys' side of the maximum: 1, 1, 1

  v16f o[TD];
#pragma unroll
  for (int td = 0; td < TD; ++td)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[td][r] = 0.f;
  float m = 0.f;                                     // running maximum of the lane's row
  bool fresh = true;                                 // the row has seen no key yet
  float l = 0.f;

  // ---- places of this lane's operands in a buffer: chunks of one row differ by an xor (and whole groups of chunks) ----
  constexpr int kGroup1 = Chunks<RC1>::kBits, kGroup2 = Chunks<RC2>::kBits, kGroupV = Chunks<RCV>::kBits;
  auto lds16 = [](uint32_t at) __attribute__((always_inline)) { return *reinterpret_cast<const __attribute__((address_space(3))) u32x4*>(at); };

  auto tile_step = [&](int j, auto MASKED, int buffer, bool prefetch) __attribute__((always_inline)) {
    constexpr bool masked = decltype(MASKED)::value;
    const Source next = source(j + 1, prefetch);
    // worked out anew for every tile: kept, they would be the registers that do not fit
    int ln = lane;
    asm volatile("" : "+v"(ln));
    const int l32 = ln & 31, hi = ln >> 5, i16 = ln & 15, half = (ln >> 4) & 1, v_row = 4 * hi + (i16 >> 2);
    const uint32_t base = lds_base + (uint32_t)(buffer * kBuffer);
    const uint32_t k_at = base + l32 * kRow1 + ((hi ^ swz1(l32)) << 4);
    const uint32_t k2_at = base + kTile1 + l32 * kRow2 + ((hi ^ Chunks<RC2>::keys(l32)) << 4);
    const uint32_t v_at = base + (SHARED ? 0 : kTile1 + kTile2) + v_row * kRowV + (((2 * half + ((i16 & 3) >> 1)) ^ swzv(v_row)) << 4) + ((i16 & 1) << 3);
    v16f s[2];
    const v16f nothing = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if constexpr (SHARED) {
      const int tt = j_last - j;
      const float t0 = (float)(tt & 255), t1 = (float)(tt >> 8);
#pragma unroll
      for (int tk = 0; tk < 2; ++tk) {
        const float at = (float)(l32 + 32 * tk);
        const uint4 k_more = make_uint4(hi ? ones : pack2<bf16_t>(at, at), hi ? ones & 0xffffu : pack2<bf16_t>(at, t0), pack2<bf16_t>(t0, t0), pack2<bf16_t>(t1, t1));
        s[tk] = mfma32x32x16<bf16_t>(k_more, q_more, nothing);
      }
    } else {
      const uint4 k_more = make_uint4(ones, ones & 0xffffu, 0u, 0u);
      s[0] = mfma32x32x16<bf16_t>(k_more, q_more, nothing);
      s[1] = mfma32x32x16<bf16_t>(k_more, q_more, nothing);
    }
    // ---- scores: fragments one step ahead of the products, a copy of the next tile behind every step ----
    constexpr int KS = KS1 + KS2;
    auto k_frag = [&](auto K, int tk) __attribute__((always_inline)) {
      constexpr int ks = decltype(K)::value, k2 = ks - KS1;
      u32x4 x;
      if constexpr (ks < KS1) x = lds16((k_at ^ (32u * (ks % (kGroup1 / 2)))) + 16 * kGroup1 * (ks / (kGroup1 / 2)) + tk * 32 * kRow1);
      else x = lds16((k2_at ^ (32u * (k2 % (kGroup2 / 2)))) + 16 * kGroup2 * (k2 / (kGroup2 / 2)) + tk * 32 * kRow2);
      return make_uint4(x[0], x[1], x[2], x[3]);
    };
    uint4 kf[2][2];
#pragma unroll
    for (int tk = 0; tk < 2; ++tk) kf[0][tk] = k_frag(std::integral_constant<int, 0>{}, tk);
    static_for<KS>([&](auto K) {
      constexpr int ks = decltype(K)::value;
      if constexpr (ks + 1 < KS) {
#pragma unroll
        for (int tk = 0; tk < 2; ++tk) kf[(ks + 1) & 1][tk] = k_frag(std::integral_constant<int, ks + 1>{}, tk);
        __builtin_amdgcn_sched_barrier(0);
      }
#pragma unroll
      for (int tk = 0; tk < 2; ++tk) s[tk] = mfma32x32x16<bf16_t>(kf[ks & 1][tk], qf[ks], s[tk]);
      if constexpr (ks < kCopies) copy(next, K, buffer ^ 1);
    });
    if constexpr (KS < kCopies)
      static_for<kCopies - KS>([&](auto C) { copy(next, std::integral_constant<int, KS + decltype(C)::value>{}, buffer ^ 1); });

    // ---- softmax, one query row per lane ----
    if constexpr (masked) {
      const int pos = pos0 + l32 - j * kWinKeys - 4 * hi, low = pos - W;         // keys low < key <= pos (relative)
#pragma unroll
      for (int tk = 0; tk < 2; ++tk)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int key = 32 * tk + 8 * (r >> 2) + (r & 3);
          if (key > pos || key <= low) s[tk][r] = -INFINITY;
        }
    }
    const float mx0 = fmaxf(s[0][15], s[1][15]);     // ordinary reads of both chains first (prefill_mfma.h)
    float mx = mx0, mx1 = mx0;
#pragma unroll
    for (int r = 0; r < 14; r += 2) {
      mx = max3(mx, s[0][r], s[0][r + 1]);
      mx1 = max3(mx1, s[1][r], s[1][r + 1]);
    }
    mx = fmaxf(max3(mx, s[0][14], s[1][14]), mx1);
    mx = max_with_lane_xor32(mx);                    // relative to the running maximum
    const bool grow = fresh ? mx > -INFINITY : mx > 8.f;
    if (KS1 > 8 ? __builtin_expect(__any(grow), 0) : __any(grow)) {
      const float d = grow ? mx : 0.f, alpha = fresh ? 1.f : fast_exp2(-d);
      l *= alpha;
#pragma unroll
      for (int td = 0; td < TD; ++td)
#pragma unroll
        for (int r = 0; r < 16; ++r) o[td][r] *= alpha;
      m += d;
      const float m0 = to_float(from_float<bf16_t>(m)), m1 = to_float(from_float<bf16_t>(m - m0)), m2 = m - m0 - m1;
      if (hi) q_more = make_uint4(pack2<bf16_t>(-m0, -m1), pack2<bf16_t>(-m2, 0.f), 0u, 0u);
#pragma unroll
      for (int tk = 0; tk < 2; ++tk)
#pragma unroll
        for (int r = 0; r < 16; ++r) s[tk][r] -= d;
      fresh = fresh && !grow;
    }
#pragma unroll
    for (int tk = 0; tk < 2; ++tk)
#pragma unroll
      for (int r = 0; r < 16; ++r) s[tk][r] = fast_exp2(s[tk][r]);

    // ---- Oᵀ += Vᵀ Pᵀ, 16 keys at a time ----
    static_for<4>([&](auto STEP) {
      constexpr int step = decltype(STEP)::value, tk = step / 2, st = step % 2;
      uint4 pf;
      pf.x = pack2<bf16_t>(s[tk][8 * st + 0], s[tk][8 * st + 1]);
      pf.y = pack2<bf16_t>(s[tk][8 * st + 2], s[tk][8 * st + 3]);
      pf.z = pack2<bf16_t>(s[tk][8 * st + 4], s[tk][8 * st + 5]);
      pf.w = pack2<bf16_t>(s[tk][8 * st + 6], s[tk][8 * st + 7]);
      l = add_pair<bf16_t>(pf.w, add_pair<bf16_t>(pf.z, add_pair<bf16_t>(pf.y, add_pair<bf16_t>(pf.x, l))));
      uint4 vf[TD];
#pragma unroll
      for (int td = 0; td < TD; ++td) {
        const uint32_t at = (v_at ^ (64u * (td % (kGroupV / 4)))) + 16 * kGroupV * (td / (kGroupV / 4));
        auto turned = [](uint32_t p) __attribute__((always_inline)) {
          return __builtin_bit_cast(uint2, __builtin_amdgcn_ds_read_tr16_b64_v4i16(reinterpret_cast<__attribute__((address_space(3))) v4s*>(p)));
        };
        const uint2 a0 = turned(at + 16 * step * kRowV), a1 = turned((SHARED ? at ^ 32u : at) + (16 * step + 8) * kRowV);
        vf[td] = make_uint4(a0.x, a0.y, a1.x, a1.y);
      }
#pragma unroll
      for (int td = 0; td < TD; ++td) o[td] = mfma32x32x16<bf16_t>(vf[td], pf, o[td]);
    });
  };

  int buffer = 0;
  for (int j = wg_first; j <= wg_last; ++j, buffer ^= 1) {
    dma_wait_all();
    __syncthreads();                                 // tile j is there; nobody reads the other buffer any more
    const bool more = j < wg_last;
    if (!active || j < j_first || j > j_last) {      // other waves' tile: this wave's share of the next copy only
      if (more) {
        const Source s = source(j + 1, true);
        static_for<kCopies>([&](auto C) { copy(s, C, buffer ^ 1); });
      }
      continue;
    }
    const bool whole = j * kWinKeys > pos0 + kWinRows - 1 - W && j * kWinKeys + kWinKeys - 1 <= pos0;
    if (KS1 <= 8 && whole) tile_step(j, std::false_type{}, buffer, more);
    else tile_step(j, std::true_type{}, buffer, more);      // (the large heads: one copy of the step, whose registers then stay put)
  }

  // ---- normalise, turn through LDS, store whole rows ----
  dma_wait_all();
  __syncthreads();
  if (!active) return;
  char* ot = lds + wave * (kWinRows * kRowV);
  {
    const float sum = sum_with_lane_xor32(l), inv = sum > 0.f ? 1.f / sum : 0.f;
#pragma unroll
    for (int td = 0; td < TD; ++td)
#pragma unroll
      for (int r4 = 0; r4 < 4; ++r4) {
        const uint2 w = make_uint2(pack2<bf16_t>(o[td][4 * r4 + 0] * inv, o[td][4 * r4 + 1] * inv), pack2<bf16_t>(o[td][4 * r4 + 2] * inv, o[td][4 * r4 + 3] * inv));
        *reinterpret_cast<uint2*>(ot + l32 * kRowV + (((4 * td + r4) ^ Chunks<RCV>::keys(l32)) << 4) + 8 * hi) = w;
      }
  }
#pragma unroll
  for (int i = 0; i < 2 * TD; ++i) {
    const int c = i * 64 + lane, row = c / RCV, p = c % RCV;
    uint4 w = *reinterpret_cast<const uint4*>(ot + row * kRowV + ((p ^ Chunks<RCV>::keys(row)) << 4));
    if (r0 + row >= seq_len) continue;
    const int64_t t = (int64_t)seq_start + r0 + row;
    if (a.gate) {
      const bf16_t* gate = reinterpret_cast<const bf16_t*>(a.gate) + t * a.gate_row + (int64_t)h * a.gate_head;
      uint4 gw;
      if (a.gate_head == 1) {
        const uint32_t two = (uint32_t)gate->bits * 0x10001u;
        gw = make_uint4(two, two, two, two);
      } else {
        gw = *reinterpret_cast<const uint4*>(gate + 8 * p);
      }
      auto gated = [](uint32_t x, uint32_t y) __attribute__((always_inline)) {
        auto sig = [](float z) __attribute__((always_inline)) { return __builtin_amdgcn_rcpf(1.f + __expf(-z)); };
        return pack2<bf16_t>(lo_to_float<bf16_t>(x) * sig(lo_to_float<bf16_t>(y)), hi_to_float<bf16_t>(x) * sig(hi_to_float<bf16_t>(y)));
      };
      w = make_uint4(gated(w.x, gw.x), gated(w.y, gw.y), gated(w.z, gw.z), gated(w.w, gw.w));
    }
    store16_stream(reinterpret_cast<bf16_t*>(a.out) + t * a.out_row + (int64_t)h * a.out_head + 8 * p, w);
  }
}

template <int KS1, int KS2, int TD, bool SHARED>
static int launch_window_prefill(const WindowPrefillArgs& a, hipStream_t s) {
  WindowPrefillArgs b = a;
  const int group = a.heads / a.kv_heads;
  b.hpw = group % 4 == 0 ? 4 : group % 2 == 0 ? 2 : 1;
  const int bm = kWinRows * (4 / b.hpw);
  b.band_shift = band_shift_for(a.total_q, a.num_seqs, bm, false);
  b.tiles_x = (int)(a.total_q / bm + (a.num_seqs <= 64 ? (int64_t)a.num_seqs << b.band_shift : a.num_seqs));
  b.heads_y = a.kv_heads * (group / b.hpw);
  b.band_bits = 1;
  while (((int64_t)1 << b.band_bits) <= a.total_q / (bm << b.band_shift) + 1) ++b.band_bits;
  const int64_t items = (int64_t)b.tiles_x * b.heads_y, span = 8 * (int64_t)kXcdChunk, blocks = (items + span - 1) / span * span;
  if (blocks > 0x7fffffff) return MVLLM_ERR_UNSUPPORTED;
  window_prefill_kernel<KS1, KS2, TD, SHARED><<<dim3((unsigned)blocks), dim3(256), 0, s>>>(b);
  return launch_status();
}

constexpr int kNoTiles = 1 << 30;      // no tiled kernel is built for the sizes
// keys of two parts and values of their own (window_prefill_latent.hip), or kNoTiles
int launch_window_prefill_parts(const WindowPrefillArgs& a, hipStream_t stream);
// keys of one part and values of their own (window_prefill_heads.hip), or kNoTiles
int launch_window_prefill_heads(const WindowPrefillArgs& a, hipStream_t stream);

}  // namespace mvllm
