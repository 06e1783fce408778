// Portions with mixed heads, bf16, heads of 32 .. 128 (talk.h).
//
// A workgroup is 16 query rows and 16 of the heads that come out, 8 waves; keys go by in tiles of 32.  A tile takes three parts:
//   raw scores of ALL heads: wave p has up to four heads of one kv head (a piece), K straight from memory as the A operand;
//   every score goes to LDS as a sum of two bf16 numbers, eight of them (four heads, both terms, or twice two heads) in 16 bytes;
//   mixing: wave w has the queries 2 w and 2 w + 1; the entries of a (query, key) are a row of the A operand whose contraction
//   index runs over (piece, term, head), against talk with every number twice, in fp32 (talk itself is bf16 in a
//   checkpoint, the scores are good to 2^-17).  A lane ends with one head and eight keys of a query: softmax, and the weights go
//   back to where the wave's own entries were;
//   O += P V: a wave has four heads of one kv head and half their columns, or two heads and all columns; V in whole rows, turned
//   by byte permutations as in talk_decode.hip.
// The entries lie so that sixteen queries with one key and sixteen keys with one query both fall into different banks.
#include "prefill_mfma.h"
#include "talk.h"

#pragma clang fp contract(off)

namespace mvllm {

constexpr int kTalkRows = 16, kTalkTile = 32;

// Eight bytes to 16 of a row, zeros past the descriptor's end.
template <int N> __device__ __forceinline__ void load_words(__amdgpu_buffer_rsrc_t rows, uint32_t at, uint32_t all, uint32_t* w) {
  if constexpr (N == 4) {
    const auto x = __builtin_amdgcn_raw_buffer_load_b128(rows, at, all, 0);
    w[0] = x[0]; w[1] = x[1]; w[2] = x[2]; w[3] = x[3];
  } else if constexpr (N == 3) {
    const auto x = __builtin_amdgcn_raw_buffer_load_b96(rows, at, all, 0);
    w[0] = x[0]; w[1] = x[1]; w[2] = x[2];
  } else if constexpr (N == 2) {
    const auto x = __builtin_amdgcn_raw_buffer_load_b64(rows, at, all, 0);
    w[0] = x[0]; w[1] = x[1];
  } else {
    w[0] = __builtin_amdgcn_raw_buffer_load_b32(rows, at, all, 0);
  }
}

// NV = dim / 32, HPP = heads of a piece (4, or 2: one step of the mixing product, whose 32 numbers are eight pieces' two heads
// and both terms), SHARE: how many neighbouring heads surely share a kv head where they are added up (1, 2 or 4).
template <int NV, int HPP, int SHARE>
__global__ __launch_bounds__(512, 2) void talk_prefill_kernel(const TalkArgs a) {
  constexpr int NS = HPP / 2;                        // steps of the mixing product
  constexpr int kEntry = 64 * NS;                    // bytes of a (query, key)
  constexpr int kBuffer = kTalkRows * kTalkTile * kEntry;
  __shared__ __attribute__((aligned(1024))) char lds[2 * kBuffer];
  __shared__ __attribute__((aligned(16))) float keep_of[16][kTalkRows];       // head, query: factor of what is accumulated
  __shared__ __attribute__((aligned(16))) int grown[8];

  // ---- work item: (tile of heads, query rows), dealt as in prefill_mfma.h ----
  const unsigned id = blockIdx.x, slot = id >> 3, xcd = id & 7, round = slot / kXcdChunk;
  const unsigned item = (round * 8 + ((xcd + round) & 7)) * kXcdChunk + slot % kXcdChunk;
  int seq_start, seq_len, row0, seq, head_tile;
  if (a.num_seqs <= 64) {
    if (!locate_banded<kTalkRows>(a.cu_q, a.num_seqs, item, a.heads_y, a.band_bits, a.band_shift, seq_start, seq_len, row0, seq, head_tile)) return;
  } else {
    if (item >= (unsigned)a.tiles_x * (unsigned)a.heads_y) return;
    head_tile = (int)(item / (unsigned)a.tiles_x);
    if (!locate_tile(a.cu_q, a.num_seqs, a.tiles_x - 1 - (int)(item % (unsigned)a.tiles_x), kTalkRows, seq_start, seq_len, row0, seq)) return;
  }
  head_tile = __builtin_amdgcn_readfirstlane(head_tile);
  seq_start = __builtin_amdgcn_readfirstlane(seq_start);
  seq_len = __builtin_amdgcn_readfirstlane(seq_len);
  row0 = __builtin_amdgcn_readfirstlane(row0);
  seq = __builtin_amdgcn_readfirstlane(seq);
  const int k_start = a.cu_k ? a.cu_k[seq] : seq_start, kv_len = a.cu_k ? a.cu_k[seq + 1] - k_start : seq_len, cached = kv_len - seq_len;
  const int32_t* table = a.tables ? a.tables + (int64_t)seq * a.table_width : nullptr;

  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), quad = lane >> 4, i16 = lane & 15;
  const int H = a.heads, G = a.kv_heads, per = a.per;
  // piece p: its kv head, first head and number of heads
  auto kv_of = [&](int p) __attribute__((always_inline)) { return (int)((unsigned)p * a.piece_magic >> 16); };
  auto first_head = [&](int p) __attribute__((always_inline)) { return kv_of(p) * per + (p - kv_of(p) * a.pieces_per_kv) * HPP; };
  auto heads_in = [&](int p) __attribute__((always_inline)) { return p < a.pieces ? min(HPP, per - (p - kv_of(p) * a.pieces_per_kv) * HPP) : 0; };

  // ---- this wave's queries (columns of the raw scores: query row i16) and its part of talk ----
  const bool scores = wave < a.pieces;
  const int own_piece = min(wave, a.pieces - 1), kv_raw = kv_of(own_piece);
  uint4 qf[HPP][NV], tf[NS];
  {
    const int64_t row = (int64_t)seq_start + min(row0 + i16, seq_len - 1);
    const int h0 = first_head(own_piece), n = heads_in(own_piece);
#pragma unroll
    for (int e = 0; e < HPP; ++e) {
      const bf16_t* q = reinterpret_cast<const bf16_t*>(a.q) + (row * H + h0 + min(e, n - 1)) * (32 * NV) + 8 * quad;
#pragma unroll
      for (int ks = 0; ks < NV; ++ks) qf[e][ks] = *reinterpret_cast<const uint4*>(q + 32 * ks);
    }
    const int h = 16 * head_tile + i16;
    const float* talk = a.talk + min(h, H - 1) * H;
    float t[NS][4];
    bool there[NS][4];
#pragma unroll
    for (int st = 0; st < NS; ++st)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int p = HPP == 4 ? 4 * st + quad : 2 * (4 * st + quad) + e / 2, in = e % HPP, g = first_head(p) + in;
        there[st][e] = h < H && in < heads_in(p);
        t[st][e] = talk[there[st][e] ? g : 0];
      }
#pragma unroll
    for (int st = 0; st < NS; ++st) {
#pragma unroll
      for (int e = 0; e < 4; ++e) t[st][e] = there[st][e] ? t[st][e] : 0.f;
      const uint32_t x = pack2<bf16_t>(t[st][0], t[st][1]), y = pack2<bf16_t>(t[st][2], t[st][3]);
      tf[st] = HPP == 4 ? make_uint4(x, y, x, y) : make_uint4(x, x, y, y);
    }
#pragma unroll
    for (int e = 1; e < HPP; ++e)
      if (e >= n) {                                  // uniform
#pragma unroll
        for (int ks = 0; ks < NV; ++ks) qf[e][ks] = make_uint4(0u, 0u, 0u, 0u);
      }
  }
  // ---- heads this wave adds up, and which of their columns: NV (or all 2 NV) blocks of sixteen ----
  constexpr int PH = SHARE == 4 ? 4 : 2, VB = SHARE == 4 ? NV : 2 * NV, VW = VB / 2;
  static_assert(VB % 2 == 0, "a lane's columns are whole words");
  const int in_tile = SHARE == 4 ? 4 * (wave >> 1) : 2 * wave, out_head = 16 * head_tile + in_tile, out_col = SHARE == 4 ? (wave & 1) * 16 * NV : 0;
  const bool live = out_head < H;
  const int kv_out = live ? out_head / per : -1;
  v4f o[PH][VB];
#pragma unroll
  for (int e = 0; e < PH; ++e)
#pragma unroll
    for (int b = 0; b < VB; ++b) o[e][b] = v4f{0.f, 0.f, 0.f, 0.f};

  // ---- places in a buffer, as LDS addresses of the first one ----
  // entry of (query i, key k): number 16 k + x, x = i ^ (k mod 16); its 16-byte parts trade places by x
  auto entry = [](int k, int x) __attribute__((always_inline)) { return (16 * k + x) * kEntry; };
  auto part = [](int p, int x) __attribute__((always_inline)) { return (NS == 2 ? p ^ (x >> 1) : p ^ (x >> 2)) << 4; };
  constexpr int kHalf = 16 * 16 * kEntry;            // between the two sixteens of keys
  const uint32_t lds_base = lds_address(lds);
  uint32_t raw_at[4], mix_at[2][NS], weight_at[PH];   // of the raw scores of keys 4 quad + r; of key i16's, queries 2 wave + qq; of this wave's heads' weights
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int x = i16 ^ (4 * quad + r);
    raw_at[r] = lds_base + entry(4 * quad + r, x) + (HPP == 4 ? part(wave, x) : part(wave >> 1, x) + 8 * (wave & 1));
  }
#pragma unroll
  for (int e = 0; e < 2; ++e) {
    const int x = i16 ^ (2 * wave + e);
#pragma unroll
    for (int st = 0; st < NS; ++st) mix_at[e][st] = lds_base + entry(i16, x) + part(4 * st + quad, x);
  }
#pragma unroll
  for (int e = 0; e < PH; ++e) weight_at[e] = lds_base + entry(in_tile + e, i16 ^ (in_tile + e)) + part(quad, i16 ^ (in_tile + e));
  // (kept whole: taken apart into what they have in common they would be more registers)
#pragma unroll
  for (int r = 0; r < 4; ++r) asm volatile("" : "+v"(raw_at[r]));
#pragma unroll
  for (int e = 0; e < PH; ++e) asm volatile("" : "+v"(weight_at[e]));
#pragma unroll
  for (int e = 0; e < 2; ++e) {
#pragma unroll
    for (int st = 0; st < NS; ++st) asm volatile("" : "+v"(mix_at[e][st]));
  }
  auto read16 = [](uint32_t at) __attribute__((always_inline)) { return __builtin_bit_cast(uint4, *reinterpret_cast<const __attribute__((address_space(3))) u32x4*>(at)); };
  auto write16 = [](uint32_t at, uint4 w) __attribute__((always_inline)) { *reinterpret_cast<__attribute__((address_space(3))) u32x4*>(at) = u32x4{w.x, w.y, w.z, w.w}; };

  float m[2] = {0.f, 0.f}, l[2] = {0.f, 0.f};        // of (head i16, query 2 wave + qq): what scores are counted from, this lane's sum

  // ---- keys and values: sixteen of them lie in one cache block; rows past the last one arrive as zeros ----
  const uint32_t row_bytes = (uint32_t)G * (64 * NV);
  const uint32_t key_at = i16 * row_bytes + kv_raw * (64 * NV) + 16 * quad, value_at = 4 * quad * row_bytes + 2 * out_col + 4 * VW * i16;
  // first row of the sixteen keys from `base` on (uniform, scalar loads)
  auto row_of = [&](int base) __attribute__((always_inline)) {
    if (!table) return (int64_t)(k_start + base);
    const int first = min(base, (kv_len - 1) & ~15), b = first / a.block_size;
    const int block = reinterpret_cast<const __attribute__((address_space(4))) int32_t*>(reinterpret_cast<uintptr_t>(table))[b];
    return (int64_t)min(max((int64_t)block, (int64_t)0), a.num_blocks - 1) * a.block_size + (first - b * a.block_size);
  };
  // (loads that bring nothing are still made: the waits count every wave's loads alike)
  auto rows_at = [&](const void* all, int base, int64_t row, bool wanted) __attribute__((always_inline)) {
    const int count = wanted ? min(kv_len - base, 16) : 0;
    const char* p = reinterpret_cast<const char*>(all) + (count > 0 ? row : 0) * (int64_t)row_bytes;
    return __builtin_amdgcn_make_buffer_rsrc(const_cast<char*>(p), 0, count > 0 ? (uint32_t)count * row_bytes : 0u, 0x00020000);
  };
  uint4 kf[2][NV];
  auto load_key = [&](__amdgpu_buffer_rsrc_t rows, int kb, int ks) __attribute__((always_inline)) {
    kf[kb][ks] = __builtin_bit_cast(uint4, __builtin_amdgcn_raw_buffer_load_b128(rows, key_at + 64 * ks, 0, 0));
  };
  uint32_t vf[2][4][VW];
  auto load_value = [&](__amdgpu_buffer_rsrc_t rows, int kv, int kb, int j) __attribute__((always_inline)) {
    load_words<VW>(rows, value_at, (uint32_t)j * row_bytes + (uint32_t)max(kv, 0) * (64 * NV), vf[kb][j]);
  };
  auto load_values = [&](int base, const int64_t* row, int kv) __attribute__((always_inline)) {
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) {
      const auto rows = rows_at(a.v, base + 16 * kb, row[kb], kv >= 0);
#pragma unroll
      for (int j = 0; j < 4; ++j) load_value(rows, kv, kb, j);
    }
  };

  const int tiles = (cached + min(row0 + kTalkRows, seq_len) - 1) / kTalkTile + 1;
  int64_t row[2] = {row_of(0), row_of(16)};
#pragma unroll
  for (int kb = 0; kb < 2; ++kb) {
    const auto rows = rows_at(a.k, 16 * kb, row[kb], scores);
#pragma unroll
    for (int ks = 0; ks < NV; ++ks) load_key(rows, kb, ks);
  }
  for (int j = 0; j < tiles; ++j) {
    const int base = j * kTalkTile;
    const uint32_t buffer = (uint32_t)(j & 1) * kBuffer;
    const bool more = j + 1 < tiles;
    const int64_t next[2] = {row_of(base + kTalkTile), row_of(base + kTalkTile + 16)};
    const __amdgpu_buffer_rsrc_t keys[2] = {rows_at(a.k, base + kTalkTile, next[0], more && scores), rows_at(a.k, base + kTalkTile + 16, next[1], more && scores)};
    // ---- raw scores, sixteen keys at a time.  Loads are spread over the tile (all at once they wait for one another): its
    // values between these products, the next one's keys while scores are packed and while weights are made ----
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) {
      const auto values = rows_at(a.v, base + 16 * kb, row[kb], live);
      v4f s[HPP];
#pragma unroll
      for (int e = 0; e < HPP; ++e) s[e] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < NV; ++ks) {
#pragma unroll
        for (int e = 0; e < HPP; ++e) s[e] = mfma16x16x32<bf16_t>(kf[kb][ks], qf[e][ks], s[e]);
        if constexpr (SHARE > 1) {
          __builtin_amdgcn_sched_barrier(0);
          if (ks < 4) load_value(values, kv_out, kb, ks);
          if (ks == NV - 1) {
#pragma unroll
            for (int j = NV; j < 4; ++j) load_value(values, kv_out, kb, j);
          }
          __builtin_amdgcn_sched_barrier(0);
        }
      }
      auto terms = [&](int e, int r, uint32_t& high, uint32_t& low) __attribute__((always_inline)) {
        high = pack2<bf16_t>(s[e][r], s[e + 1][r]);
        low = pack2<bf16_t>(s[e][r] - lo_to_float<bf16_t>(high), s[e + 1][r] - hi_to_float<bf16_t>(high));
      };
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        uint4 w;
        terms(0, r, w.x, w.z);
        if constexpr (HPP == 4) {
          terms(2, r, w.y, w.w);
          write16(raw_at[r] + buffer + kb * kHalf, w);
        } else {
          *reinterpret_cast<__attribute__((address_space(3))) uint64_t*>(raw_at[r] + buffer + kb * kHalf) = (uint64_t)w.z << 32 | w.x;
        }
        if (kb == 1 && r < NV) load_key(keys[0], 0, r);
        __builtin_amdgcn_sched_barrier(0);
      }
    }
    workgroup_barrier();
    // ---- the wave's two queries: mixed scores (counted from the running maximum, which the sums start with), weights ----
    {
      v4f s[2][2];
#pragma unroll
      for (int qq = 0; qq < 2; ++qq) {
        uint4 in[2][NS];
#pragma unroll
        for (int st = 0; st < NS; ++st)
#pragma unroll
          for (int kb = 0; kb < 2; ++kb) in[kb][st] = read16(mix_at[qq][st] + buffer + kb * kHalf);
#pragma unroll
        for (int kb = 0; kb < 2; ++kb) s[qq][kb] = v4f{-m[qq], -m[qq], -m[qq], -m[qq]};
#pragma unroll
        for (int st = 0; st < NS; ++st)
#pragma unroll
          for (int kb = 0; kb < 2; ++kb) s[qq][kb] = mfma16x16x32<bf16_t>(in[kb][st], tf[st], s[qq][kb]);
      }
#pragma unroll
      for (int qq = 0; qq < 2; ++qq) {
        const int pos = cached + row0 + 2 * wave + qq - base;       // of the query, counted from the tile's first key
        if (pos < kTalkTile - 1) {
#pragma unroll
          for (int kb = 0; kb < 2; ++kb)
#pragma unroll
            for (int r = 0; r < 4; ++r)
              if (16 * kb + 4 * quad + r > pos) s[qq][kb][r] = -INFINITY;
        }
      }
      uint32_t w[2][4];
      float sum[2];
      auto weigh = [&](int qq) __attribute__((always_inline)) {
        sum[qq] = 0.f;
#pragma unroll
        for (int kb = 0; kb < 2; ++kb)
#pragma unroll
          for (int r = 0; r < 4; r += 2) {
            w[qq][2 * kb + r / 2] = pack2<bf16_t>(fast_exp2(s[qq][kb][r]), fast_exp2(s[qq][kb][r + 1]));
            sum[qq] = add_pair<bf16_t>(w[qq][2 * kb + r / 2], sum[qq]);
          }
      };
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int qq = 0; qq < 2; ++qq) {
        weigh(qq);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int ks = qq * ((NV + 1) / 2); ks < (qq ? NV : (NV + 1) / 2); ++ks) load_key(keys[1], 1, ks);
        __builtin_amdgcn_sched_barrier(0);
      }
      // weights are made anew, from the true maximum, in the first tile and where a lane's share of a row has become large
      float keep[2] = {1.f, 1.f};
      const bool again = j == 0 || __any(fmaxf(sum[0], sum[1]) > 4096.f);
      if (again) {
#pragma unroll
        for (int qq = 0; qq < 2; ++qq) {
          float top = fmaxf(fmaxf(fmaxf(s[qq][0][0], s[qq][0][1]), fmaxf(s[qq][0][2], s[qq][0][3])), fmaxf(fmaxf(s[qq][1][0], s[qq][1][1]), fmaxf(s[qq][1][2], s[qq][1][3])));
          top = fmaxf(top, __shfl_xor(top, 16, 64));
          top = fmaxf(top, __shfl_xor(top, 32, 64));
          const float d = j == 0 ? top : fmaxf(top, 0.f);
          keep[qq] = j == 0 ? 0.f : fast_exp2(-d);
          m[qq] += d;
          l[qq] *= keep[qq];
#pragma unroll
          for (int kb = 0; kb < 2; ++kb)
#pragma unroll
            for (int r = 0; r < 4; ++r) s[qq][kb][r] -= d;
          weigh(qq);
        }
      }
      if (quad < 2) keep_of[i16][2 * wave + quad] = quad ? keep[1] : keep[0];
      if (lane == 0) grown[wave] = again && j > 0;
      // head i16's weights go to the entry of (query, key i16): keys 4 quad .. + 3 of both sixteens
#pragma unroll
      for (int qq = 0; qq < 2; ++qq) {
        l[qq] += sum[qq];
        write16(mix_at[qq][0] + buffer, make_uint4(w[qq][0], w[qq][1], w[qq][2], w[qq][3]));
      }
    }
    workgroup_barrier();
    // ---- the wave's heads ----
    {
      const int4 g0 = reinterpret_cast<const int4*>(grown)[0], g1 = reinterpret_cast<const int4*>(grown)[1];
      if (__builtin_amdgcn_readfirstlane(g0.x | g0.y | g0.z | g0.w | g1.x | g1.y | g1.z | g1.w)) {
#pragma unroll
        for (int e = 0; e < PH; ++e) {
          const float4 f = *reinterpret_cast<const float4*>(&keep_of[in_tile + e][4 * quad]);
#pragma unroll
          for (int b = 0; b < VB; ++b) o[e][b] = v4f{o[e][b][0] * f.x, o[e][b][1] * f.y, o[e][b][2] * f.z, o[e][b][3] * f.w};
        }
      }
      uint4 pf[PH];
#pragma unroll
      for (int e = 0; e < PH; ++e) pf[e] = read16(weight_at[e] + buffer);
      auto add = [&](auto FIRST, auto COUNT) __attribute__((always_inline)) {
        constexpr int first = decltype(FIRST)::value, count = decltype(COUNT)::value;
#pragma unroll
        for (int d = 0; d < VW; ++d) {
          auto turned = [&](uint32_t sel) __attribute__((always_inline)) {
            return make_uint4(__builtin_amdgcn_perm(vf[0][1][d], vf[0][0][d], sel), __builtin_amdgcn_perm(vf[0][3][d], vf[0][2][d], sel),
                              __builtin_amdgcn_perm(vf[1][1][d], vf[1][0][d], sel), __builtin_amdgcn_perm(vf[1][3][d], vf[1][2][d], sel));
          };
          const uint4 lo = turned(0x05040100u), hi = turned(0x07060302u);
#pragma unroll
          for (int e = first; e < first + count; ++e) {
            o[e][2 * d] = mfma16x16x32<bf16_t>(pf[e], lo, o[e][2 * d]);
            o[e][2 * d + 1] = mfma16x16x32<bf16_t>(pf[e], hi, o[e][2 * d + 1]);
          }
        }
      };
      using std::integral_constant;
      if constexpr (SHARE > 1) {
        add(integral_constant<int, 0>{}, integral_constant<int, PH>{});
      } else {
        if (live) {
          load_values(base, row, kv_out);
          add(integral_constant<int, 0>{}, integral_constant<int, 1>{});
        }
        if (out_head + 1 < H) {
          load_values(base, row, (out_head + 1) / per);
          add(integral_constant<int, 1>{}, integral_constant<int, 1>{});
        }
      }
    }
    row[0] = next[0];
    row[1] = next[1];
  }

  // ---- sums to where the heads are, normalise, store whole rows ----
#pragma unroll
  for (int qq = 0; qq < 2; ++qq) {
    l[qq] += __shfl_xor(l[qq], 16, 64);
    l[qq] += __shfl_xor(l[qq], 32, 64);
    const int h = 16 * head_tile + i16;
    if (a.sinks && h < H) l[qq] = add_sink(l[qq], m[qq], a.sinks[h]);
  }
  workgroup_barrier();                               // the last factors have been read
  if (quad < 2) {
    const float sum = quad ? l[1] : l[0];
    keep_of[i16][2 * wave + quad] = sum > 0.f ? 1.f / sum : 0.f;
  }
  workgroup_barrier();
#pragma unroll
  for (int e = 0; e < PH; ++e) {
    if (out_head + e >= H) continue;
    const float4 f4 = *reinterpret_cast<const float4*>(&keep_of[in_tile + e][4 * quad]);
    const float f[4] = {f4.x, f4.y, f4.z, f4.w};
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = row0 + 4 * quad + r;
      if (row >= seq_len) continue;
      int64_t t = (int64_t)seq_start + row;
      if (a.out_rows) t = a.out_rows[t];
      uint32_t* p = reinterpret_cast<uint32_t*>(reinterpret_cast<bf16_t*>(a.out) + t * a.out_row + (out_head + e) * a.out_head + out_col + 2 * VW * i16);
      uint32_t w[VW];
#pragma unroll
      for (int d = 0; d < VW; ++d) w[d] = pack2<bf16_t>(o[e][2 * d][r] * f[r], o[e][2 * d + 1][r] * f[r]);
      if constexpr (VW % 2 == 0) {
#pragma unroll
        for (int d = 0; d < VW; d += 2) *reinterpret_cast<uint2*>(p + d) = make_uint2(w[d], w[d + 1]);
      } else {
#pragma unroll
        for (int d = 0; d < VW; ++d) p[d] = w[d];
      }
    }
  }
}

template <int NV, int HPP>
static int launch_talk_prefill_as(const TalkArgs& a, unsigned blocks, hipStream_t s) {
  const dim3 grid(blocks), block(512);
  if constexpr (NV % 2 == 0) {
    if (a.per % 4 == 0) {
      talk_prefill_kernel<NV, HPP, 4><<<grid, block, 0, s>>>(a);
      return launch_status();
    }
  }
  if (a.per % 2 == 0) talk_prefill_kernel<NV, HPP, 2><<<grid, block, 0, s>>>(a);
  else talk_prefill_kernel<NV, HPP, 1><<<grid, block, 0, s>>>(a);
  return launch_status();
}

int launch_talk_prefill(const TalkArgs& a, hipStream_t s) {
  const int most = TalkPieces(a.heads, a.kv_heads, 2).count <= 8 ? 2 : 4;      // heads per piece: eight waves, a piece each
  const TalkPieces pieces(a.heads, a.kv_heads, most);
  if (pieces.count > 8 || (int64_t)a.kv_heads * a.dim * 32 > (1 << 24)) return kNotBuilt;
  TalkArgs b = a;
  b.per = a.heads / a.kv_heads;
  b.pieces = pieces.count;
  b.pieces_per_kv = pieces.per_kv;
  b.piece_magic = 65536u / (unsigned)pieces.per_kv + 1u;
  b.band_shift = band_shift_for(a.total_q, a.num_seqs, kTalkRows, a.tables != nullptr);
  b.tiles_x = (int)(a.total_q / kTalkRows + (a.num_seqs <= 64 ? (int64_t)a.num_seqs << b.band_shift : a.num_seqs));
  b.heads_y = (a.heads + 15) / 16;
  b.band_bits = 1;
  while (((int64_t)1 << b.band_bits) <= a.total_q / (kTalkRows << b.band_shift) + 1) ++b.band_bits;
  const int64_t items = (int64_t)b.tiles_x * b.heads_y, span = 8 * (int64_t)kXcdChunk, blocks = (items + span - 1) / span * span;
  if (blocks > 0x7fffffff) return MVLLM_ERR_UNSUPPORTED;
  switch (a.dim) {
    case 32: return most == 2 ? launch_talk_prefill_as<1, 2>(b, (unsigned)blocks, s) : launch_talk_prefill_as<1, 4>(b, (unsigned)blocks, s);
    case 64: return most == 2 ? launch_talk_prefill_as<2, 2>(b, (unsigned)blocks, s) : launch_talk_prefill_as<2, 4>(b, (unsigned)blocks, s);
    case 96: return most == 2 ? launch_talk_prefill_as<3, 2>(b, (unsigned)blocks, s) : launch_talk_prefill_as<3, 4>(b, (unsigned)blocks, s);
    case 128: return most == 2 ? launch_talk_prefill_as<4, 2>(b, (unsigned)blocks, s) : launch_talk_prefill_as<4, 4>(b, (unsigned)blocks, s);
    default: return kNotBuilt;
  }
}

}  // namespace mvllm
