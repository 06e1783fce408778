// Single query rows with mixed heads over a paged cache, bf16, heads of 32 .. 128 (talk.h).
//
// A workgroup is a (share of the keys, row) with all heads; wave = (kv head, one of KS groups of keys), 32 keys at a time.
//   raw scores: K from global straight into the A operand (key = lane % 16), its heads as columns;
//   the waves of a key group exchange them through LDS in fp32 (one barrier per 32 keys, two buffers);
//   mixed scores: v_mfma_f32_16x16x4_f32 over the heads, exact products, each wave for its own heads only, which leaves a
//   lane with one head and four keys of each 16, the A operand of
//   O += P V: V loaded in whole rows, a lane's consecutive dims, and turned into the B operand by byte permutations (column
//   lane % 16 of block n is dim 2 NV (lane % 16) + n).
// The next keys and values are on their way while these are worked on.
#include "talk.h"

#pragma clang fp contract(off)

namespace mvllm {

constexpr int kTalkKeys = 32;          // keys per step of a wave
constexpr size_t kMostLds = 64 * 1024;
constexpr int kRawRow = 48;            // floats of a head's raw scores: four heads' rows fall into different banks

__device__ __forceinline__ uint32_t low_halves(uint32_t a, uint32_t b) { return __builtin_amdgcn_perm(b, a, 0x05040100u); }
__device__ __forceinline__ uint32_t high_halves(uint32_t a, uint32_t b) { return __builtin_amdgcn_perm(b, a, 0x07060302u); }

struct TalkDecodeLayout {              // dynamic LDS, in floats
  int quads, talk_row, talk, raw, box, total;
  __host__ __device__ TalkDecodeLayout(int heads, int kv_heads, int dim, int tiles, int splits) {
    quads = (heads + 3) / 4;
    talk_row = heads + 32;             // columns past the last head stay zeros
    talk = 4 * quads * talk_row;
    raw = 2 * splits * 4 * quads * kRawRow;
    box = splits > 1 ? kv_heads * tiles * (dim / 16) * 64 * 4 + kv_heads * tiles * 32 : 0;
    total = talk + (raw > box ? raw : box);
  }
};

// NV = dim / 32, HT = 16-head tiles of a kv head's query heads.
template <int NV, int HT>
__global__ __launch_bounds__(512, 2) void talk_decode_kernel(const TalkArgs a, int splits) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int H = a.heads, G = a.kv_heads, per = H / G;
  const TalkDecodeLayout at(H, G, 32 * NV, HT, splits);
  float* talk = lds;
  float* raw = lds + at.talk;
  const int part = blockIdx.x, row = blockIdx.y;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), quad = lane >> 4, i16 = lane & 15;
  const int kv = wave % G, split = wave / G;

  // ---- the row's share of keys ----
  const int n = (int)min(max(a.lens[row], (int64_t)0), (int64_t)a.table_width * a.block_size);
  const int chunks = (n + 63) / 64, share = (chunks + a.parts - 1) / a.parts;
  const int k0 = min(part * share * 64, n), k1 = min(k0 + share * 64, n);
  const int32_t* table = a.tables + (int64_t)row * a.table_width;

  for (int i = tid; i < at.talk; i += blockDim.x) {
    const int g = i / at.talk_row, h = i - g * at.talk_row;
    talk[i] = g < H && h < H ? a.talk[h * H + g] : 0.f;
  }
  for (int i = tid; i < at.raw; i += blockDim.x) raw[i] = 0.f;       // rows of heads that are not there

  uint4 qf[HT][NV];
#pragma unroll
  for (int ht = 0; ht < HT; ++ht) {
    const int in = 16 * ht + i16;
    const bf16_t* q = reinterpret_cast<const bf16_t*>(a.q) + ((int64_t)row * H + kv * per + min(in, per - 1)) * (32 * NV) + 8 * quad;
#pragma unroll
    for (int ks = 0; ks < NV; ++ks) qf[ht][ks] = *reinterpret_cast<const uint4*>(q + 32 * ks);
  }
  v4f o[HT][2 * NV];
  float m[HT], l[HT];
#pragma unroll
  for (int ht = 0; ht < HT; ++ht) {
    m[ht] = -INFINITY;
    l[ht] = 0.f;
#pragma unroll
    for (int b = 0; b < 2 * NV; ++b) o[ht][b] = v4f{0.f, 0.f, 0.f, 0.f};
  }

  uint4 kf[2][NV];
  uint32_t vf[2][4][NV];
  // sixteen keys from `base` on lie in one block; keys past the last one are read inside that block or repeat it
  auto rows_of = [&](int base) __attribute__((always_inline)) {
    const int first = min(base, (k1 - 1) & ~15), b = first / a.block_size;
    const int64_t block = min(max((int64_t)table[b], (int64_t)0), a.num_blocks - 1);
    return block * a.block_size + (first - b * a.block_size);
  };
  auto load = [&](int base) __attribute__((always_inline)) {
    const int64_t row_bytes = (int64_t)G * (64 * NV);
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) {
      const int64_t r = rows_of(base + 16 * kb);
      const char* k = reinterpret_cast<const char*>(a.k) + (r + i16) * row_bytes + kv * (64 * NV) + 16 * quad;
#pragma unroll
      for (int ks = 0; ks < NV; ++ks) kf[kb][ks] = load16_stream(k + 64 * ks);
      const char* v = reinterpret_cast<const char*>(a.v) + (r + 4 * quad) * row_bytes + kv * (64 * NV) + 4 * NV * i16;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const uint32_t* p = reinterpret_cast<const uint32_t*>(v + j * row_bytes);
        if constexpr (NV == 4) {
          const uint4 w = load16_stream(p);
          vf[kb][j][0] = w.x; vf[kb][j][1] = w.y; vf[kb][j][2] = w.z; vf[kb][j][3] = w.w;
        } else {
#pragma unroll
          for (int d = 0; d < NV; ++d) vf[kb][j][d] = __builtin_nontemporal_load(p + d);
        }
      }
    }
  };

  const int step = splits * kTalkKeys, steps = (k1 - k0 + step - 1) / step;
  if (steps > 0) load(k0 + split * kTalkKeys);
  __syncthreads();
  for (int it = 0; it < steps; ++it) {
    const int base = k0 + it * step + split * kTalkKeys;
    float* own = raw + ((it & 1) * splits + split) * 4 * at.quads * kRawRow;
    // ---- raw scores of the wave's kv head ----
#pragma unroll
    for (int kb = 0; kb < 2; ++kb)
#pragma unroll
      for (int ht = 0; ht < HT; ++ht) {
        v4f s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < NV; ++ks) s = mfma16x16x32<bf16_t>(kf[kb][ks], qf[ht][ks], s);
        if (16 * ht + i16 < per)
          *reinterpret_cast<float4*>(own + (kv * per + 16 * ht + i16) * kRawRow + 16 * kb + 4 * quad) = make_float4(s[0], s[1], s[2], s[3]);
      }
    uint32_t vb[2][4][NV];                           // this step's values; the registers of the loads belong to the next one
#pragma unroll
    for (int kb = 0; kb < 2; ++kb)
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int d = 0; d < NV; ++d) vb[kb][j][d] = vf[kb][j][d];
    if (it + 1 < steps) load(base + step);
    workgroup_barrier();                             // the other kv heads' scores are there; loads stay in flight
    // ---- the wave's heads, mixed ----
#pragma unroll
    for (int ht = 0; ht < HT; ++ht) {
      v4f s[2] = {v4f{0.f, 0.f, 0.f, 0.f}, v4f{0.f, 0.f, 0.f, 0.f}};
      const float* t_at = talk + quad * at.talk_row + kv * per + 16 * ht + i16;
      const float* s_at = own + quad * kRawRow + i16;
      for (int g4 = 0; g4 < at.quads; ++g4) {
        const float t = t_at[4 * g4 * at.talk_row];
#pragma unroll
        for (int kb = 0; kb < 2; ++kb) s[kb] = __builtin_amdgcn_mfma_f32_16x16x4f32(s_at[4 * g4 * kRawRow + 16 * kb], t, s[kb], 0, 0, 0);
      }
      float most = -INFINITY;
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          if (base + 16 * kb + 4 * quad + r >= k1) s[kb][r] = -INFINITY;
          most = fmaxf(most, s[kb][r]);
        }
      most = fmaxf(most, __shfl_xor(most, 16, 64));
      most = fmaxf(most, __shfl_xor(most, 32, 64));
      // the running maximum moves only when it grows by more than 2^8 (or from nothing)
      if (__any(most > m[ht] + 8.f || (m[ht] == -INFINITY && most > -INFINITY))) {
        const float m_new = fmaxf(m[ht], most), keep = m[ht] == -INFINITY ? 0.f : fast_exp2(m[ht] - m_new);
        m[ht] = m_new;
        l[ht] *= keep;
        float f[4];                                  // of the heads the accumulators hold
#pragma unroll
        for (int r = 0; r < 4; ++r) f[r] = __shfl(keep, 4 * quad + r, 64);
#pragma unroll
        for (int b = 0; b < 2 * NV; ++b)
#pragma unroll
          for (int r = 0; r < 4; ++r) o[ht][b][r] *= f[r];
      }
      float p[2][4];
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          p[kb][r] = m[ht] == -INFINITY ? 0.f : fast_exp2(s[kb][r] - m[ht]);
          l[ht] += p[kb][r];
        }
      const uint4 w = make_uint4(pack2<bf16_t>(p[0][0], p[0][1]), pack2<bf16_t>(p[0][2], p[0][3]), pack2<bf16_t>(p[1][0], p[1][1]), pack2<bf16_t>(p[1][2], p[1][3]));
#pragma unroll
      for (int d = 0; d < NV; ++d) {
        const uint4 lo = make_uint4(low_halves(vb[0][0][d], vb[0][1][d]), low_halves(vb[0][2][d], vb[0][3][d]),
                                    low_halves(vb[1][0][d], vb[1][1][d]), low_halves(vb[1][2][d], vb[1][3][d]));
        const uint4 hi = make_uint4(high_halves(vb[0][0][d], vb[0][1][d]), high_halves(vb[0][2][d], vb[0][3][d]),
                                    high_halves(vb[1][0][d], vb[1][1][d]), high_halves(vb[1][2][d], vb[1][3][d]));
        o[ht][2 * d] = mfma16x16x32<bf16_t>(w, lo, o[ht][2 * d]);
        o[ht][2 * d + 1] = mfma16x16x32<bf16_t>(w, hi, o[ht][2 * d + 1]);
      }
    }
  }
#pragma unroll
  for (int ht = 0; ht < HT; ++ht) {
    l[ht] += __shfl_xor(l[ht], 16, 64);
    l[ht] += __shfl_xor(l[ht], 32, 64);
  }

  // ---- the key groups of a kv head meet in LDS, one after the other ----
  if (splits > 1) {
    float4* box = reinterpret_cast<float4*>(raw) + kv * HT * 2 * NV * 64;
    float2* ml = reinterpret_cast<float2*>(raw + G * HT * 2 * NV * 64 * 4) + kv * HT * 16;
    for (int other = 1; other < splits; ++other) {
      __syncthreads();
      if (split == other) {
#pragma unroll
        for (int ht = 0; ht < HT; ++ht) {
#pragma unroll
          for (int b = 0; b < 2 * NV; ++b) box[(ht * 2 * NV + b) * 64 + lane] = make_float4(o[ht][b][0], o[ht][b][1], o[ht][b][2], o[ht][b][3]);
          if (quad == 0) ml[ht * 16 + i16] = make_float2(m[ht], l[ht]);
        }
      }
      __syncthreads();
      if (split == 0) {
#pragma unroll
        for (int ht = 0; ht < HT; ++ht) {
          const float2 x = ml[ht * 16 + i16];
          const float m_new = fmaxf(m[ht], x.x);
          const float mine = m[ht] == -INFINITY ? 0.f : fast_exp2(m[ht] - m_new), theirs = x.x == -INFINITY ? 0.f : fast_exp2(x.x - m_new);
          float f[4], g[4];
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            f[r] = __shfl(mine, 4 * quad + r, 64);
            g[r] = __shfl(theirs, 4 * quad + r, 64);
          }
#pragma unroll
          for (int b = 0; b < 2 * NV; ++b) {
            const float4 w = box[(ht * 2 * NV + b) * 64 + lane];
            o[ht][b] = v4f{o[ht][b][0] * f[0] + w.x * g[0], o[ht][b][1] * f[1] + w.y * g[1], o[ht][b][2] * f[2] + w.z * g[2], o[ht][b][3] * f[3] + w.w * g[3]};
          }
          l[ht] = l[ht] * mine + x.y * theirs;
          m[ht] = m_new;
        }
      }
    }
  }
  if (split != 0) return;
#pragma unroll
  for (int ht = 0; ht < HT; ++ht) {
    const int own_head = kv * per + 16 * ht + i16;
    if (a.parts > 1 && quad == 0 && 16 * ht + i16 < per) a.part_ml[((int64_t)row * a.parts + part) * H + own_head] = make_float2(m[ht], l[ht]);
    float sum = l[ht];
    if (a.sinks && a.parts == 1 && 16 * ht + i16 < per) sum = add_sink(sum, m[ht], a.sinks[own_head]);
    const float inv = sum > 0.f ? 1.f / sum : 0.f;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int in = 16 * ht + 4 * quad + r, h = kv * per + in;
      const float f = __shfl(inv, 4 * quad + r, 64);
      if (in >= per) continue;
      if (a.parts > 1) {
        float* p = a.part_o + (((int64_t)row * a.parts + part) * H + h) * (32 * NV) + 2 * NV * i16;
#pragma unroll
        for (int b = 0; b < 2 * NV; b += 2) *reinterpret_cast<float2*>(p + b) = make_float2(o[ht][b][r], o[ht][b + 1][r]);
      } else {
        uint32_t* p = reinterpret_cast<uint32_t*>(reinterpret_cast<bf16_t*>(a.out) + row * a.out_row + h * a.out_head + 2 * NV * i16);
#pragma unroll
        for (int d = 0; d < NV; ++d) p[d] = pack2<bf16_t>(o[ht][2 * d][r] * f, o[ht][2 * d + 1][r] * f);
      }
    }
  }
}

template <int NV>
static int launch_talk_decode_as(const TalkArgs& a, int rows, hipStream_t s) {
  const int tiles = (a.heads / a.kv_heads + 15) / 16;
  auto bytes_of = [&](int splits) { return (size_t)TalkDecodeLayout(a.heads, a.kv_heads, a.dim, tiles, splits).total * sizeof(float); };
  int splits = 8 / a.kv_heads;
  while (splits > 1 && bytes_of(splits) > kMostLds) --splits;
  const size_t bytes = bytes_of(splits);
  if (bytes > kMostLds) return kNotBuilt;
  const dim3 grid((unsigned)a.parts, (unsigned)rows), block((unsigned)(64 * a.kv_heads * splits));
  if (tiles == 1) talk_decode_kernel<NV, 1><<<grid, block, bytes, s>>>(a, splits);
  else talk_decode_kernel<NV, 2><<<grid, block, bytes, s>>>(a, splits);
  return launch_status();
}

int launch_talk_decode(const TalkArgs& a, int rows, hipStream_t s) {
  int st;
  switch (a.dim) {
    case 32: st = launch_talk_decode_as<1>(a, rows, s); break;
    case 64: st = launch_talk_decode_as<2>(a, rows, s); break;
    case 96: st = launch_talk_decode_as<3>(a, rows, s); break;
    case 128: st = launch_talk_decode_as<4>(a, rows, s); break;
    default: return kNotBuilt;
  }
  if (st != MVLLM_OK || a.parts == 1) return st;
  LatentDecodeArgs b = {};             // what the pass that joins shares reads
  b.out = a.out; b.out_row = a.out_row; b.out_head = a.out_head; b.part_o = a.part_o; b.part_ml = a.part_ml; b.heads = a.heads;
  b.kv_heads = a.kv_heads; b.values = a.dim; b.parts = a.parts; b.sinks = a.sinks;
  latent_merge_kernel<bf16_t, true><<<dim3((unsigned)(((int64_t)rows * a.heads + 3) / 4)), dim3(256), 0, s>>>(b, rows);
  return launch_status();
}

}  // namespace mvllm
