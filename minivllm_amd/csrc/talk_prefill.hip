// Portions with mixed heads, bf16, heads of 32 .. 128 (talk.h).
//
// A workgroup is 16 query rows and 16 of the heads that come out, 8 waves; keys go by in tiles of 32.  A tile takes three parts:
//   raw scores of ALL heads: wave p has four heads of one kv head (a piece), K straight from memory as the A operand; every
//   score goes to LDS as a sum of two bf16 numbers, eight of them (four heads, both terms) in one entry of 16 bytes;
//   mixing: wave w has the queries 2 w and 2 w + 1; the entries of a (query, key) are a row of the A operand whose contraction
//   index runs over (piece, term, head), against talk with every number twice, in fp32 (talk itself is bf16 in a
//   checkpoint, the scores are good to 2^-17).  A lane ends with one head and eight keys of a query: softmax, and the weights go
//   back to where the wave's own entries were;
//   O += P V: wave w has the heads 2 w and 2 w + 1, V in whole rows, turned by byte permutations as in talk_decode.hip.
// The entries lie so that sixteen queries with one key and sixteen keys with one query both fall into different banks.
#include "prefill_mfma.h"
#include "talk.h"

#pragma clang fp contract(off)

namespace mvllm {

constexpr int kTalkRows = 16, kTalkTile = 32;

// NV = dim / 32, NS = steps of four pieces, PAIR: heads 2 n and 2 n + 1 share a kv head.
template <int NV, int NS, bool PAIR>
__global__ __launch_bounds__(512, 2) void talk_prefill_kernel(const TalkArgs a) {
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
  const int H = a.heads, G = a.kv_heads, per = H / G;
  const TalkPieces pieces(H, G);
  auto first_head = [&](int p) __attribute__((always_inline)) { return p / pieces.per_kv * per + p % pieces.per_kv * 4; };
  auto heads_in = [&](int p) __attribute__((always_inline)) { return p < pieces.count ? min(4, per - p % pieces.per_kv * 4) : 0; };

  if (pieces.count < 4 * NS) {                       // entries of pieces that are not there: any finite number will do
    for (int i = tid; i < 2 * kBuffer / 16; i += 512) *reinterpret_cast<uint4*>(lds + 16 * i) = make_uint4(0u, 0u, 0u, 0u);
    __syncthreads();
  }

  // ---- this wave's queries (columns of the raw scores: query row i16) and its part of talk ----
  const bool scores = wave < pieces.count;
  const int kv_raw = min(wave, pieces.count - 1) / pieces.per_kv;
  uint4 qf[4][NV];
  {
    const int64_t row = (int64_t)seq_start + min(row0 + i16, seq_len - 1);
    const int h0 = first_head(min(wave, pieces.count - 1)), n = heads_in(wave);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const bf16_t* q = reinterpret_cast<const bf16_t*>(a.q) + (row * H + h0 + min(e, max(n - 1, 0))) * (32 * NV) + 8 * quad;
#pragma unroll
      for (int ks = 0; ks < NV; ++ks) qf[e][ks] = e < n ? *reinterpret_cast<const uint4*>(q + 32 * ks) : make_uint4(0u, 0u, 0u, 0u);
    }
  }
  uint4 tf[NS];
#pragma unroll
  for (int st = 0; st < NS; ++st) {
    const int p = 4 * st + quad, n = heads_in(p), h0 = p < pieces.count ? first_head(p) : 0, h = 16 * head_tile + i16;
    float t[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) t[e] = h < H && e < n ? a.talk[h * H + h0 + e] : 0.f;
    const uint32_t x = pack2<bf16_t>(t[0], t[1]), y = pack2<bf16_t>(t[2], t[3]);
    tf[st] = make_uint4(x, y, x, y);
  }
  // ---- places in a buffer ----
  // entry of (query i, key k): number 16 k + x, x = i ^ (k mod 16); a piece's 16 bytes trade places by x
  auto entry = [](int k, int x) __attribute__((always_inline)) { return (16 * k + x) * kEntry; };
  auto part = [](int p, int x) __attribute__((always_inline)) { return (NS == 2 ? p ^ (x >> 1) : p ^ (x >> 2)) << 4; };

  // ---- heads this wave adds up ----
  const int out_head = 16 * head_tile + 2 * wave;
  const bool live[2] = {out_head < H, out_head + 1 < H};
  const int kv_out[2] = {min(out_head, H - 1) / per, min(out_head + 1, H - 1) / per};
  v4f o[2][2 * NV];
#pragma unroll
  for (int e = 0; e < 2; ++e)
#pragma unroll
    for (int b = 0; b < 2 * NV; ++b) o[e][b] = v4f{0.f, 0.f, 0.f, 0.f};
  float m[2] = {-INFINITY, -INFINITY}, l[2] = {0.f, 0.f};      // of (head i16, query 2 wave + qq)

  // ---- keys and values: sixteen of them lie in one cache block; past the last one some row that exists ----
  const int64_t row_bytes = (int64_t)G * (64 * NV);
  auto rows_at = [&](int base) __attribute__((always_inline)) {
    const int first = min(base, (kv_len - 1) & ~15);
    if (!table) return (int64_t)(k_start + first);
    const int b = first / a.block_size;
    return (int64_t)min(max((int64_t)table[b], (int64_t)0), a.num_blocks - 1) * a.block_size + (first - b * a.block_size);
  };
  auto most_rows = [&](int base) __attribute__((always_inline)) { return table ? 15 : min(15, kv_len - 1 - min(base, (kv_len - 1) & ~15)); };
  uint4 kf[2][NV];
  auto load_keys = [&](int base) __attribute__((always_inline)) {
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) {
      const char* k = reinterpret_cast<const char*>(a.k) + (rows_at(base + 16 * kb) + min(i16, most_rows(base + 16 * kb))) * row_bytes + kv_raw * (64 * NV) + 16 * quad;
#pragma unroll
      for (int ks = 0; ks < NV; ++ks) kf[kb][ks] = *reinterpret_cast<const uint4*>(k + 64 * ks);
    }
  };
  uint32_t vf[2][4][NV];
  auto load_values = [&](int base, int kv) __attribute__((always_inline)) {
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) {
      const int64_t first = rows_at(base + 16 * kb);
      const int most = most_rows(base + 16 * kb);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const char* v = reinterpret_cast<const char*>(a.v) + (first + min(4 * quad + j, most)) * row_bytes + kv * (64 * NV) + 4 * NV * i16;
        if constexpr (NV == 4) {
          const uint4 w = *reinterpret_cast<const uint4*>(v);
          vf[kb][j][0] = w.x; vf[kb][j][1] = w.y; vf[kb][j][2] = w.z; vf[kb][j][3] = w.w;
        } else if constexpr (NV == 2) {
          const uint2 w = *reinterpret_cast<const uint2*>(v);
          vf[kb][j][0] = w.x; vf[kb][j][1] = w.y;
        } else {
#pragma unroll
          for (int d = 0; d < NV; ++d) vf[kb][j][d] = reinterpret_cast<const uint32_t*>(v)[d];
        }
      }
    }
  };

  const int tiles = (cached + min(row0 + kTalkRows, seq_len) - 1) / kTalkTile + 1;
  if (scores) load_keys(0);
  if (PAIR && live[0]) load_values(0, kv_out[0]);
  for (int j = 0; j < tiles; ++j) {
    const int base = j * kTalkTile;
    char* buffer = lds + (j & 1) * kBuffer;
    // ---- raw scores ----
    if (scores) {
      v4f s[2][4];
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int e = 0; e < 4; ++e) s[kb][e] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < NV; ++ks)
#pragma unroll
        for (int kb = 0; kb < 2; ++kb)
#pragma unroll
          for (int e = 0; e < 4; ++e) s[kb][e] = mfma16x16x32<bf16_t>(kf[kb][ks], qf[e][ks], s[kb][e]);
      if (j + 1 < tiles) load_keys(base + kTalkTile);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int x = i16 ^ (4 * quad + r);
        char* at = buffer + entry(4 * quad + r, x) + part(wave, x);
#pragma unroll
        for (int kb = 0; kb < 2; ++kb) {
          const uint32_t h01 = pack2<bf16_t>(s[kb][0][r], s[kb][1][r]), h23 = pack2<bf16_t>(s[kb][2][r], s[kb][3][r]);
          const uint32_t l01 = pack2<bf16_t>(s[kb][0][r] - lo_to_float<bf16_t>(h01), s[kb][1][r] - hi_to_float<bf16_t>(h01));
          const uint32_t l23 = pack2<bf16_t>(s[kb][2][r] - lo_to_float<bf16_t>(h23), s[kb][3][r] - hi_to_float<bf16_t>(h23));
          *reinterpret_cast<uint4*>(at + 16 * kb * 16 * kEntry) = make_uint4(h01, h23, l01, l23);
        }
      }
    }
    workgroup_barrier();
    // ---- the wave's two queries: mixed scores, weights ----
    {
      v4f s[2][2];
#pragma unroll
      for (int qq = 0; qq < 2; ++qq) {
        const int x = i16 ^ (2 * wave + qq);
        const char* at = buffer + entry(i16, x);
#pragma unroll
        for (int kb = 0; kb < 2; ++kb) {
          s[qq][kb] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int st = 0; st < NS; ++st)
            s[qq][kb] = mfma16x16x32<bf16_t>(*reinterpret_cast<const uint4*>(at + 16 * kb * 16 * kEntry + part(4 * st + quad, x)), tf[st], s[qq][kb]);
        }
      }
      float most[2];
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
        most[qq] = fmaxf(fmaxf(fmaxf(s[qq][0][0], s[qq][0][1]), fmaxf(s[qq][0][2], s[qq][0][3])), fmaxf(fmaxf(s[qq][1][0], s[qq][1][1]), fmaxf(s[qq][1][2], s[qq][1][3])));
      }
      // a running maximum moves only when it grows by more than 2^8 (or from nothing)
      float keep[2] = {1.f, 1.f};
      const bool grow = __any(most[0] > m[0] + 8.f || most[1] > m[1] + 8.f);
      if (grow) {
#pragma unroll
        for (int qq = 0; qq < 2; ++qq) {
          float top = fmaxf(most[qq], __shfl_xor(most[qq], 16, 64));
          top = fmaxf(top, __shfl_xor(top, 32, 64));
          const float m_new = top > m[qq] + 8.f ? top : m[qq];
          keep[qq] = m_new == m[qq] ? 1.f : fast_exp2(m[qq] - m_new);
          m[qq] = m_new;
          l[qq] *= keep[qq];
        }
      }
      if (quad < 2) keep_of[i16][2 * wave + quad] = quad ? keep[1] : keep[0];
      if (lane == 0) grown[wave] = grow;
#pragma unroll
      for (int qq = 0; qq < 2; ++qq) {
        uint32_t w[4];
#pragma unroll
        for (int kb = 0; kb < 2; ++kb)
#pragma unroll
          for (int r = 0; r < 4; r += 2) {
            w[2 * kb + r / 2] = pack2<bf16_t>(fast_exp2(s[qq][kb][r] - m[qq]), fast_exp2(s[qq][kb][r + 1] - m[qq]));
            l[qq] = add_pair<bf16_t>(w[2 * kb + r / 2], l[qq]);
          }
        // head i16's weights in the entry of (query, key i16): keys 4 quad .. + 3 of both sixteens
        const int x = i16 ^ (2 * wave + qq);
        *reinterpret_cast<uint4*>(buffer + entry(i16, x) + part(quad, x)) = make_uint4(w[0], w[1], w[2], w[3]);
      }
    }
    workgroup_barrier();
    // ---- the wave's two heads ----
    {
      const int4 g0 = reinterpret_cast<const int4*>(grown)[0], g1 = reinterpret_cast<const int4*>(grown)[1];
      if (__builtin_amdgcn_readfirstlane(g0.x | g0.y | g0.z | g0.w | g1.x | g1.y | g1.z | g1.w)) {
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          const float4 f = *reinterpret_cast<const float4*>(&keep_of[2 * wave + e][4 * quad]);
#pragma unroll
          for (int b = 0; b < 2 * NV; ++b) o[e][b] = v4f{o[e][b][0] * f.x, o[e][b][1] * f.y, o[e][b][2] * f.z, o[e][b][3] * f.w};
        }
      }
      uint4 pf[2];
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const int h = 2 * wave + e, x = i16 ^ h;
        pf[e] = *reinterpret_cast<const uint4*>(buffer + entry(h, x) + part(quad, x));
      }
      auto add = [&](auto FIRST, auto COUNT) __attribute__((always_inline)) {
        constexpr int first = decltype(FIRST)::value, count = decltype(COUNT)::value;
#pragma unroll
        for (int d = 0; d < NV; ++d) {
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
      if constexpr (PAIR) {
        if (live[0]) {
          add(integral_constant<int, 0>{}, integral_constant<int, 2>{});
          if (j + 1 < tiles) load_values(base + kTalkTile, kv_out[0]);
        }
      } else {
        if (live[0]) {
          load_values(base, kv_out[0]);
          add(integral_constant<int, 0>{}, integral_constant<int, 1>{});
        }
        if (live[1]) {
          load_values(base, kv_out[1]);
          add(integral_constant<int, 1>{}, integral_constant<int, 1>{});
        }
      }
    }
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
  for (int e = 0; e < 2; ++e) {
    if (!live[e]) continue;
    const float4 f4 = *reinterpret_cast<const float4*>(&keep_of[2 * wave + e][4 * quad]);
    const float f[4] = {f4.x, f4.y, f4.z, f4.w};
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = row0 + 4 * quad + r;
      if (row >= seq_len) continue;
      int64_t t = (int64_t)seq_start + row;
      if (a.out_rows) t = a.out_rows[t];
      uint32_t* p = reinterpret_cast<uint32_t*>(reinterpret_cast<bf16_t*>(a.out) + t * a.out_row + (out_head + e) * a.out_head + 2 * NV * i16);
      uint32_t w[NV];
#pragma unroll
      for (int d = 0; d < NV; ++d) w[d] = pack2<bf16_t>(o[e][2 * d][r] * f[r], o[e][2 * d + 1][r] * f[r]);
      if constexpr (NV == 4) {
        *reinterpret_cast<uint2*>(p) = make_uint2(w[0], w[1]);
        *reinterpret_cast<uint2*>(p + 2) = make_uint2(w[2], w[3]);
      } else {
#pragma unroll
        for (int d = 0; d < NV; ++d) p[d] = w[d];
      }
    }
  }
}

template <int NV>
static int launch_talk_prefill_as(const TalkArgs& a, unsigned blocks, hipStream_t s) {
  const bool few = TalkPieces(a.heads, a.kv_heads).count <= 4, pair = a.heads / a.kv_heads % 2 == 0;
  const dim3 grid(blocks), block(512);
  if (few && pair) talk_prefill_kernel<NV, 1, true><<<grid, block, 0, s>>>(a);
  else if (few) talk_prefill_kernel<NV, 1, false><<<grid, block, 0, s>>>(a);
  else if (pair) talk_prefill_kernel<NV, 2, true><<<grid, block, 0, s>>>(a);
  else talk_prefill_kernel<NV, 2, false><<<grid, block, 0, s>>>(a);
  return launch_status();
}

int launch_talk_prefill(const TalkArgs& a, hipStream_t s) {
  if (TalkPieces(a.heads, a.kv_heads).count > 8) return kNotBuilt;
  TalkArgs b = a;
  b.band_shift = band_shift_for(a.total_q, a.num_seqs, kTalkRows, a.tables != nullptr);
  b.tiles_x = (int)(a.total_q / kTalkRows + (a.num_seqs <= 64 ? (int64_t)a.num_seqs << b.band_shift : a.num_seqs));
  b.heads_y = (a.heads + 15) / 16;
  b.band_bits = 1;
  while (((int64_t)1 << b.band_bits) <= a.total_q / (kTalkRows << b.band_shift) + 1) ++b.band_bits;
  const int64_t items = (int64_t)b.tiles_x * b.heads_y, span = 8 * (int64_t)kXcdChunk, blocks = (items + span - 1) / span * span;
  if (blocks > 0x7fffffff) return MVLLM_ERR_UNSUPPORTED;
  switch (a.dim) {
    case 32: return launch_talk_prefill_as<1>(b, (unsigned)blocks, s);
    case 64: return launch_talk_prefill_as<2>(b, (unsigned)blocks, s);
    case 96: return launch_talk_prefill_as<3>(b, (unsigned)blocks, s);
    case 128: return launch_talk_prefill_as<4>(b, (unsigned)blocks, s);
    default: return kNotBuilt;
  }
}

}  // namespace mvllm
