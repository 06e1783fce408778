// Matrix memory in blocks of 64 rows on the matrix unit, for portions of many rows (bf16 inputs).
// With the gates of the mLSTM (mlstm.hip), F_t the running sum of the log forget gates, a_s = i_s - F_s and
// M_t = max(m, max_{s <= t} a_s):
//     m_t   = F_t + M_t                                  (m: the running maximum in front of the block)
//     num_t = exp(m - M_t) S^T q_t + sum_{s <= t} exp(a_s - M_t) (q_t . k_s) v_s
//     n.q_t = exp(m - M_t) n . q_t + sum_{s <= t} exp(a_s - M_t) (q_t . k_s)
//     S'    = exp(m - M_L) S + sum_s exp(a_s - M_L) k_s v_s^T,   n' likewise with k_s alone
// Without gates, S <- decay S + k v^T with a constant of the head, the same forms hold with exp(m - M_t) = decay^(t + 1),
// exp(a_s - M_t) = decay^(t - s), exp(a_s - M_L) = decay^(L - 1 - s), and there is neither n nor m.
// q, k and v are bf16 and enter exactly; what is not (S, the weighted scores, the weighted values) enters a product as
// the sum of two bf16 numbers, so the products are good to 2^-17 and S, n and m stay fp32.
//
// Workgroup = (segment, head, 32 kWaves value columns), kWaves waves of 32 columns each; S lives in the waves' accumulator
// registers ([dim x 32] per wave) and is the B operand of its own product with q as it lies there: the accumulator layout
// of v_mfma_f32_32x32x16 (row 8 (r / 4) + 4 (l / 32) + r % 4, column l % 32) is its operand layout under a permutation of
// the contraction index, k-slot (l / 32, e) of a 16-wide step = 8 (e / 4) + 4 (l / 32) + e % 4, which the other operand
// follows: two 8-byte reads instead of one of 16, or the transposing loads, which deliver exactly that order.
//
// A long portion is cut into segments of whole blocks that run side by side: kStateOnly first computes every segment's
// own contribution to the state from nothing, memory_combine_kernel turns those into the state in front of every segment,
// and the second pass computes the outputs from there.  Grids follow from host arguments alone.
#pragma once
#include "prefill_tiles.h"

namespace mvllm {

constexpr int kBlock = 64;           // rows per block

struct MemoryChunkArgs {
  float* num;                // [T, H, vdim]
  float* den;                // [T, H]
  float* m_next;             // [entries, H]
  const bf16_t* proj;        // [T, proj_stride]
  const float* gates;        // [T, 2 H]
  float* s_state;            // [slots, H, dim, vdim]
  float* n_state;            // [slots, H, dim]
  const float* m_state;      // [slots, H]
  const int32_t* cu;         // [entries + 1]
  const int32_t* slot;       // [entries]
  const int64_t* positions;
  const int32_t* segments;   // [num_segments, 4]: entry, first row, rows, flags (1: first of its entry, 2: last, 4: only)
  float* ws_s;               // [num_segments, H, dim, vdim]
  float* ws_n;               // [num_segments, H, dim]
  float* ws_m;               // [num_segments, H]: maximum
  float* ws_f;               // [num_segments, H]: sum of the log forget gates
  int64_t proj_stride;
  int num_segments, heads, dim, vdim;
  float q_scale, floor;
  const float* log_decay;    // [H], without gates
  int silu;                  // q, k and v are taken through z * sigmoid(z)
};

// eight packed values through z * sigmoid(z), rounded again
__device__ __forceinline__ uint4 silu8(uint4 w) {
  uint32_t x[4] = {w.x, w.y, w.z, w.w};
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const float a = lo_to_float<bf16_t>(x[i]), b = hi_to_float<bf16_t>(x[i]);
    x[i] = pack2<bf16_t>(a * __builtin_amdgcn_rcpf(1.0f + __expf(-a)), b * __builtin_amdgcn_rcpf(1.0f + __expf(-b)));
  }
  return make_uint4(x[0], x[1], x[2], x[3]);
}

__device__ __forceinline__ uint4 load16(__amdgpu_buffer_rsrc_t rows, uint32_t offset) {
  return __builtin_bit_cast(uint4, __builtin_amdgcn_raw_buffer_load_b128(rows, offset, 0, 0));
}

// x = hi + lo with both bf16, eight values at a time as operand fragments
struct Split8 { uint4 hi, lo; };
__device__ __forceinline__ Split8 split8(const float* x) {
  uint32_t h[4], l[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    h[i] = pack2<bf16_t>(x[2 * i], x[2 * i + 1]);
    l[i] = pack2<bf16_t>(x[2 * i] - lo_to_float<bf16_t>(h[i]), x[2 * i + 1] - hi_to_float<bf16_t>(h[i]));
  }
  return {make_uint4(h[0], h[1], h[2], h[3]), make_uint4(l[0], l[1], l[2], l[3])};
}

template <int DIMP, int kWaves, bool kStateOnly, bool kGates>
__global__ __launch_bounds__(64 * kWaves, DIMP == 256 ? 1 : 2) void memory_chunk_kernel(const MemoryChunkArgs a) {
  constexpr int kThreads = 64 * kWaves;
  constexpr int VT = 32 * kWaves;                  // value columns of the workgroup
  constexpr int kQRow = DIMP + 8, kVRow = VT + 8, kPRow = kBlock + 8;   // row lengths in LDS (elements): 16-byte skew
  constexpr int kTD = DIMP / 32;                   // 32-dim tiles of S
  constexpr int kQLoads = kBlock * DIMP / 8 / kThreads, kVLoads = kBlock * VT / 8 / kThreads;
  __shared__ __attribute__((aligned(16))) uint16_t qs[kStateOnly ? 8 : kBlock * kQRow];
  __shared__ __attribute__((aligned(16))) uint16_t ks[kBlock * kQRow];
  __shared__ __attribute__((aligned(16))) uint16_t vs[kBlock * kVRow];
  __shared__ __attribute__((aligned(16))) uint16_t ph[kStateOnly ? 8 : kBlock * kPRow], pl[kStateOnly ? 8 : kBlock * kPRow];
  __shared__ float sc_a[kBlock], sc_M[kBlock], sc_in[kBlock], sc_w[kBlock], sc_floor[kBlock];
  __shared__ float n_lds[kGates ? DIMP : 1], n_part[kGates ? kThreads * 2 : 1];

  const int seg = blockIdx.x, h = blockIdx.y, tile = blockIdx.z;
  const int entry = a.segments[4 * seg], row0 = a.segments[4 * seg + 1], rows = a.segments[4 * seg + 2];
  const int flags = a.segments[4 * seg + 3];
  const int slot = a.slot[entry];
  if (rows <= 0 || slot < 0 || (kStateOnly && (flags & 2))) return;     // the last segment's contribution is not needed
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l32 = lane & 31, hi = lane >> 5, i16 = lane & 15, half = (lane >> 4) & 1;
  const int dim = a.dim, vdim = a.vdim, H = a.heads;
  const int col = tile * VT + 32 * wave + l32;     // this lane's value column
  const bool has_col = col < vdim;
  const bool n_owner = kGates && tile == 0;
  const float log_decay = kGates ? 0.f : a.log_decay[h];

  // ---- the state in front of the segment ----
  v16f s[kTD];
  float m;
  const float* s_in = nullptr;
  const float* n_in = nullptr;
  if constexpr (kStateOnly) {
    m = -INFINITY;
  } else if (flags & 4) {                           // an entry in one piece: straight from its slot
    const bool fresh = a.positions[row0] == 0;
    m = !kGates || fresh ? 0.f : a.m_state[(int64_t)slot * H + h];
    if (!fresh) {
      s_in = a.s_state + ((int64_t)slot * H + h) * dim * vdim;
      if constexpr (kGates) n_in = a.n_state + ((int64_t)slot * H + h) * dim;
    }
  } else {
    m = kGates ? a.ws_m[(int64_t)seg * H + h] : 0.f;
    s_in = a.ws_s + ((int64_t)seg * H + h) * dim * vdim;
    if constexpr (kGates) n_in = a.ws_n + ((int64_t)seg * H + h) * dim;
  }
  // bounds-checked: rows past dim and columns past vdim (and everything without a state) arrive as zeros
  const uint32_t s_bytes = (uint32_t)(dim * vdim) * 4u;
  const uint32_t s_first = has_col ? (uint32_t)(4 * hi * vdim + col) * 4u : 0x80000000u;
  {
    const auto state = __builtin_amdgcn_make_buffer_rsrc(const_cast<float*>(s_in), 0, s_in != nullptr ? s_bytes : 0u, 0x00020000);
    static_for<kTD>([&](auto TD) {
      constexpr int td = decltype(TD)::value;
#pragma unroll
      for (int r = 0; r < 16; ++r)
        s[td][r] = __uint_as_float(__builtin_amdgcn_raw_buffer_load_b32(state, s_first + (uint32_t)((32 * td + 8 * (r >> 2) + (r & 3)) * vdim) * 4u, 0, 0));
      __builtin_amdgcn_sched_barrier(0);
    });
  }
  if (n_owner)
    for (int d = tid; d < DIMP; d += kThreads) n_lds[d] = n_in != nullptr && d < dim ? n_in[d] : 0.f;

  // ---- loads of a block: 16 bytes per thread and step, zeros past the rows, dims and columns that exist ----
  uint4 qr[kStateOnly ? 1 : kQLoads], kr[kQLoads], vr[kVLoads];
  float gate_i = -INFINITY, gate_f = 0.f;           // of row `lane`, in every wave
  const bf16_t* qg = a.proj + (int64_t)h * dim;
  const bf16_t* kg = a.proj + (int64_t)(H + h) * dim;
  const bf16_t* vg = a.proj + (int64_t)2 * H * dim + (int64_t)h * vdim + tile * VT;
  constexpr int kQStep = kThreads / (DIMP / 8), kVStep = kThreads / (VT / 8);      // rows between a thread's loads
  const int q_r = tid / (DIMP / 8), q_d = (tid % (DIMP / 8)) * 8, v_r = tid / (VT / 8), v_d = (tid % (VT / 8)) * 8;
  // bounds-checked: rows past the segment's end and columns past dim / vdim arrive as zeros
  const uint32_t pitch_in = (uint32_t)a.proj_stride * 2u;
  const uint32_t q_first = q_d < dim ? (uint32_t)q_r * pitch_in + (uint32_t)q_d * 2u : 0x80000000u;
  const uint32_t v_first = tile * VT + v_d < vdim ? (uint32_t)v_r * pitch_in + (uint32_t)v_d * 2u : 0x80000000u;
  auto fetch = [&](int at) __attribute__((always_inline)) {
    const int64_t base = (int64_t)(row0 + at) * a.proj_stride;
    const uint32_t reach = (uint32_t)(min(kBlock, rows - at) - 1) * pitch_in;
    auto rows_of = [&](const bf16_t* p, int cols) {
      return __builtin_amdgcn_make_buffer_rsrc(const_cast<bf16_t*>(p + base), 0, reach + (uint32_t)cols * 2u, 0x00020000);
    };
    uint32_t q_off = q_first, v_off = v_first;
    asm volatile("" : "+v"(q_off), "+v"(v_off));    // (offsets of all loads kept across the loop would not fit the registers)
    const auto k_rows = rows_of(kg, dim), v_rows = rows_of(vg, vdim - tile * VT);
    if constexpr (!kStateOnly) {
      const auto q_rows = rows_of(qg, dim);
#pragma unroll
      for (int i = 0; i < kQLoads; ++i) qr[i] = load16(q_rows, q_off + (uint32_t)(i * kQStep) * pitch_in);
    }
#pragma unroll
    for (int i = 0; i < kQLoads; ++i) kr[i] = load16(k_rows, q_off + (uint32_t)(i * kQStep) * pitch_in);
#pragma unroll
    for (int i = 0; i < kVLoads; ++i) vr[i] = load16(v_rows, v_off + (uint32_t)(i * kVStep) * pitch_in);
    if constexpr (kGates) {
      const bool live = at + lane < rows;
      const float* g = a.gates + (int64_t)(row0 + at + (live ? lane : 0)) * 2 * H;
      gate_i = live ? g[h] : -INFINITY;
      gate_f = live ? g[H + h] : 0.f;
    }
  };
  fetch(0);

  float f_total = 0.f;                              // kStateOnly: sum of the log forget gates so far
  for (int at = 0; at < rows; at += kBlock) {
    // ---- registers -> LDS; the block's scalars ----
    if constexpr (!kGates) {
      if (a.silu) {
#pragma unroll
        for (int i = 0; i < kQLoads; ++i) {
          if constexpr (!kStateOnly) qr[i] = silu8(qr[i]);
          kr[i] = silu8(kr[i]);
        }
#pragma unroll
        for (int i = 0; i < kVLoads; ++i) vr[i] = silu8(vr[i]);
      }
    }
#pragma unroll
    for (int i = 0; i < kQLoads; ++i) {
      if constexpr (!kStateOnly) *reinterpret_cast<uint4*>(&qs[(q_r + i * kQStep) * kQRow + q_d]) = qr[i];
      *reinterpret_cast<uint4*>(&ks[(q_r + i * kQStep) * kQRow + q_d]) = kr[i];
    }
#pragma unroll
    for (int i = 0; i < kVLoads; ++i) *reinterpret_cast<uint4*>(&vs[(v_r + i * kVStep) * kVRow + v_d]) = vr[i];
    float decay;                                    // of the state over the block
    if constexpr (kGates) {
      float F = gate_f;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const float t = __shfl_up(F, o, 64);
        if (lane >= o) F += t;
      }
      const float av = gate_i - F;
      float M = fmaxf(av, m);
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const float t = __shfl_up(M, o, 64);
        if (lane >= o) M = fmaxf(M, t);
      }
      const float M_last = __shfl(M, 63, 64), F_last = __shfl(F, 63, 64);
      decay = __expf(m - M_last);
      if (wave == 0) {
        sc_a[lane] = av;
        sc_M[lane] = M;
        sc_in[lane] = __expf(m - M);
        sc_w[lane] = __expf(av - M_last);
        sc_floor[lane] = __expf(-(F + M));
      }
      f_total += F_last;
      m = F_last + M_last;
    } else {
      // weights exp((t - s) log decay): the same differences of two scalars, none of them positive
      const int n = min(kBlock, rows - at);
      decay = __expf((float)n * log_decay);
      if (wave == 0) {
        sc_a[lane] = -(float)lane * log_decay;
        sc_M[lane] = -(float)lane * log_decay;
        sc_in[lane] = __expf((float)(lane + 1) * log_decay);
        sc_w[lane] = lane < n ? __expf((float)(n - 1 - lane) * log_decay) : 0.f;
      }
    }
    __syncthreads();
    if (at + kBlock < rows) fetch(at + kBlock);     // the next block's rows, on their way during this one

    v16f o[2];
    if constexpr (!kStateOnly) {
      // ---- weighted scores: the three 32 x 32 quarters at and below the diagonal ----
      static_for<3>([&](auto Q) {
        constexpr int quarter = decltype(Q)::value;
        if (quarter % kWaves != wave) return;
        constexpr int rt = quarter == 0 ? 0 : 1, ct = quarter == 2 ? 1 : 0;
        v16f p;
#pragma unroll
        for (int r = 0; r < 16; ++r) p[r] = 0.f;
#pragma unroll
        for (int st = 0; st < DIMP / 16; ++st) {
          const uint4 qa = *reinterpret_cast<const uint4*>(&qs[(32 * rt + l32) * kQRow + 16 * st + 8 * hi]);
          const uint4 kb = *reinterpret_cast<const uint4*>(&ks[(32 * ct + l32) * kQRow + 16 * st + 8 * hi]);
          p = mfma32x32x16<bf16_t>(qa, kb, p);
          if (st % 4 == 3) __builtin_amdgcn_sched_barrier(0);       // keep the operands of later steps in LDS until then
        }
        // key column sx of the lane, rows 32 rt + 4 hi + 8 (r / 4) + r % 4; past the diagonal the weight is exp(-inf)
        const int sx = 32 * ct + l32, t0 = 32 * rt + 4 * hi;
        int past = l32 - 4 * hi;                    // on the diagonal: rows `up` below it are past the key
        asm volatile("" : "+v"(past));              // (sixteen lane masks kept across the loop would not fit the registers)
        const float as = sc_a[sx];
        uint16_t* hp = &ph[t0 * kPRow + sx];
        uint16_t* lp = &pl[t0 * kPRow + sx];
        const float* Mp = &sc_M[t0];
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          constexpr float kNever = -INFINITY;
          const int up = 8 * (r >> 2) + (r & 3);
          const float arg = rt == ct && past > up ? kNever : as - Mp[up];
          const float x = p[r] * (a.q_scale * __expf(arg));
          const bf16_t top = from_float<bf16_t>(x);
          hp[up * kPRow] = top.bits;
          lp[up * kPRow] = from_float<bf16_t>(x - to_float(top)).bits;
        }
      });
      // ---- what the state in front of the block contributes ----
#pragma unroll
      for (int rt = 0; rt < 2; ++rt)
#pragma unroll
        for (int r = 0; r < 16; ++r) o[rt][r] = 0.f;
      static_for<kTD>([&](auto TD) {
        constexpr int td = decltype(TD)::value;
        static_for<2>([&](auto ST) {
          constexpr int st = decltype(ST)::value;
          float x[8];
#pragma unroll
          for (int e = 0; e < 8; ++e) x[e] = s[td][8 * st + e];
          const Split8 b = split8(x);
#pragma unroll
          for (int rt = 0; rt < 2; ++rt) {
            const uint16_t* p = &qs[(32 * rt + l32) * kQRow + 32 * td + 16 * st + 4 * hi];
            const uint2 lo = *reinterpret_cast<const uint2*>(p), up = *reinterpret_cast<const uint2*>(p + 8);
            const uint4 qa = make_uint4(lo.x, lo.y, up.x, up.y);
            o[rt] = mfma32x32x16<bf16_t>(qa, b.hi, o[rt]);
            o[rt] = mfma32x32x16<bf16_t>(qa, b.lo, o[rt]);
          }
          __builtin_amdgcn_sched_barrier(0);
        });
      });
#pragma unroll
      for (int rt = 0; rt < 2; ++rt)
#pragma unroll
        for (int r = 0; r < 16; ++r) o[rt][r] *= sc_in[32 * rt + 8 * (r >> 2) + 4 * hi + (r & 3)] * a.q_scale;
    }
    __builtin_amdgcn_sched_barrier(0);
    // this wave's 64 x 32 values as operand fragments (k-slot order as above)
    uint4 vf[4];
    {
      const uint16_t* p = &vs[(4 * hi + (i16 >> 2)) * kVRow + 32 * wave + 16 * half + 4 * (i16 & 3)];
#pragma unroll
      for (int st = 0; st < 4; ++st) {
        const v4s x0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) v4s*)(p + 16 * st * kVRow));
        const v4s x1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) v4s*)(p + (16 * st + 8) * kVRow));
        const uint2 y0 = __builtin_bit_cast(uint2, x0), y1 = __builtin_bit_cast(uint2, x1);
        vf[st] = make_uint4(y0.x, y0.y, y1.x, y1.y);
      }
    }
    if constexpr (!kStateOnly) {
      __syncthreads();                              // the weighted scores are complete
#pragma unroll
      for (int rt = 0; rt < 2; ++rt)
#pragma unroll
        for (int st = 0; st < 2 * (rt + 1); ++st) {
          const int at_p = (32 * rt + l32) * kPRow + 16 * st + 4 * hi;
          const uint2 h0 = *reinterpret_cast<const uint2*>(&ph[at_p]), h1 = *reinterpret_cast<const uint2*>(&ph[at_p + 8]);
          const uint2 l0 = *reinterpret_cast<const uint2*>(&pl[at_p]), l1 = *reinterpret_cast<const uint2*>(&pl[at_p + 8]);
          o[rt] = mfma32x32x16<bf16_t>(make_uint4(h0.x, h0.y, h1.x, h1.y), vf[st], o[rt]);
          o[rt] = mfma32x32x16<bf16_t>(make_uint4(l0.x, l0.y, l1.x, l1.y), vf[st], o[rt]);
          __builtin_amdgcn_sched_barrier(0);
        }
    }
    // ---- the state behind the block ----
    Split8 wv[4];
#pragma unroll
    for (int st = 0; st < 4; ++st) {
      const uint32_t w[4] = {vf[st].x, vf[st].y, vf[st].z, vf[st].w};
      float x[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float g = sc_w[16 * st + 8 * (e >> 2) + 4 * hi + (e & 3)];
        x[e] = g * (e & 1 ? hi_to_float<bf16_t>(w[e >> 1]) : lo_to_float<bf16_t>(w[e >> 1]));
      }
      wv[st] = split8(x);
    }
    static_for<kTD>([&](auto TD) {
      constexpr int td = decltype(TD)::value;
#pragma unroll
      for (int r = 0; r < 16; ++r) s[td][r] *= decay;
      const uint16_t* p = &ks[(4 * hi + (i16 >> 2)) * kQRow + 32 * td + 16 * half + 4 * (i16 & 3)];
#pragma unroll
      for (int st = 0; st < 4; ++st) {
        const v4s x0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) v4s*)(p + 16 * st * kQRow));
        const v4s x1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) v4s*)(p + (16 * st + 8) * kQRow));
        const uint2 y0 = __builtin_bit_cast(uint2, x0), y1 = __builtin_bit_cast(uint2, x1);
        const uint4 kf = make_uint4(y0.x, y0.y, y1.x, y1.y);
        s[td] = mfma32x32x16<bf16_t>(kf, wv[st].hi, s[td]);
        s[td] = mfma32x32x16<bf16_t>(kf, wv[st].lo, s[td]);
      }
      __builtin_amdgcn_sched_barrier(0);
    });
    // ---- normaliser and n: the head's first workgroup ----
    if constexpr (kGates) if (n_owner) {
      if constexpr (!kStateOnly) {
        constexpr int kPer = kThreads / kBlock;     // threads per row: 2 or 4
        const int t = tid / kPer, part = tid % kPer;
        float nq = 0.f, sum = 0.f;
        for (int d = 8 * part; d < DIMP; d += 8 * kPer) {
          const uint4 q4 = *reinterpret_cast<const uint4*>(&qs[t * kQRow + d]);
          const uint32_t w[4] = {q4.x, q4.y, q4.z, q4.w};
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            nq = fmaf(lo_to_float<bf16_t>(w[e]), n_lds[d + 2 * e], nq);
            nq = fmaf(hi_to_float<bf16_t>(w[e]), n_lds[d + 2 * e + 1], nq);
          }
        }
        nq *= sc_in[t] * a.q_scale;
        for (int x = 8 * part; x <= t; x += 8 * kPer) {
          const uint4 h4 = *reinterpret_cast<const uint4*>(&ph[t * kPRow + x]), l4 = *reinterpret_cast<const uint4*>(&pl[t * kPRow + x]);
          const uint32_t wh[4] = {h4.x, h4.y, h4.z, h4.w}, wl[4] = {l4.x, l4.y, l4.z, l4.w};
#pragma unroll
          for (int e = 0; e < 4; ++e)
            sum += (lo_to_float<bf16_t>(wh[e]) + lo_to_float<bf16_t>(wl[e])) + (hi_to_float<bf16_t>(wh[e]) + hi_to_float<bf16_t>(wl[e]));
        }
        nq += sum;
#pragma unroll
        for (int x = 1; x < kPer; x <<= 1) nq += __shfl_xor(nq, x, 64);
        if (part == 0 && at + t < rows) a.den[(int64_t)(row0 + at + t) * H + h] = fmaxf(fabsf(nq), sc_floor[t]) + a.floor;
      }
      // thread: one pair of dims, one share of the rows
      constexpr int kPairs = DIMP / 2, kShares = kThreads / kPairs > 0 ? kThreads / kPairs : 1, kSweeps = (kPairs + kThreads - 1) / kThreads;
#pragma unroll
      for (int sw = 0; sw < kSweeps; ++sw) {
        const int pair = (tid + sw * kThreads) % kPairs, share = kSweeps > 1 ? 0 : tid / kPairs;
        float x0 = 0.f, x1 = 0.f;
        for (int t = share; t < kBlock; t += kShares) {
          const uint32_t w = *reinterpret_cast<const uint32_t*>(&ks[t * kQRow + 2 * pair]);
          x0 = fmaf(sc_w[t], lo_to_float<bf16_t>(w), x0);
          x1 = fmaf(sc_w[t], hi_to_float<bf16_t>(w), x1);
        }
        n_part[2 * (share * kPairs + pair)] = x0;
        n_part[2 * (share * kPairs + pair) + 1] = x1;
        static_assert(kSweeps == 1, "one pair of dims per thread");
      }
      __syncthreads();                              // n has been read, the shares are there (uniform: the whole workgroup)
      for (int d = tid; d < DIMP; d += kThreads) {
        float x = 0.f;
        for (int i = 0; i < kShares; ++i) x += n_part[2 * (i * kPairs) + d];
        n_lds[d] = fmaf(decay, n_lds[d], x);
      }
    }
    if constexpr (!kStateOnly) {
      // bounds-checked stores: rows past the segment and columns past vdim are dropped
      uint32_t pitch = (uint32_t)(H * vdim) * 4u;
      asm volatile("" : "+s"(pitch));
      const int n_rows = min(kBlock, rows - at);
      const auto rsrc = __builtin_amdgcn_make_buffer_rsrc(a.num + ((int64_t)(row0 + at) * H + h) * vdim, 0,
                                                          (uint32_t)(n_rows - 1) * pitch + (uint32_t)vdim * 4u, 0x00020000);
      uint32_t voff = has_col ? (uint32_t)(4 * hi) * pitch + (uint32_t)col * 4u : 0x80000000u;
      asm volatile("" : "+v"(voff));                // (32 offsets kept across the loop would not fit the registers)
#pragma unroll
      for (int rt = 0; rt < 2; ++rt)
#pragma unroll
        for (int r = 0; r < 16; ++r)
          __builtin_amdgcn_raw_buffer_store_b32(__float_as_uint(o[rt][r]), rsrc, voff + (uint32_t)(32 * rt + 8 * (r >> 2) + (r & 3)) * pitch, 0, 2 /* nt */);
    }
    __syncthreads();                                // everybody is done with this block's LDS
  }

  // ---- the state behind the segment: contribution -> workspace (kStateOnly), the last one -> the slot ----
  if (!kStateOnly && !(flags & 2)) return;
  float* s_out = kStateOnly ? a.ws_s + ((int64_t)seg * H + h) * dim * vdim : a.s_state + ((int64_t)slot * H + h) * dim * vdim;
  const auto state = __builtin_amdgcn_make_buffer_rsrc(s_out, 0, s_bytes, 0x00020000);
  uint32_t s_pitch = (uint32_t)vdim * 4u;
  asm volatile("" : "+s"(s_pitch));
  static_for<kTD>([&](auto TD) {
    constexpr int td = decltype(TD)::value;
#pragma unroll
    for (int r = 0; r < 16; ++r)
      __builtin_amdgcn_raw_buffer_store_b32(__float_as_uint(s[td][r]), state, s_first + (uint32_t)(32 * td + 8 * (r >> 2) + (r & 3)) * s_pitch, 0, 0);
    __builtin_amdgcn_sched_barrier(0);
  });
  if constexpr (kGates) if (n_owner) {
    float* n_out = kStateOnly ? a.ws_n + ((int64_t)seg * H + h) * dim : a.n_state + ((int64_t)slot * H + h) * dim;
    for (int d = tid; d < dim; d += kThreads) n_out[d] = n_lds[d];
    if (tid == 0) {
      if constexpr (kStateOnly) {
        a.ws_m[(int64_t)seg * H + h] = m;
        a.ws_f[(int64_t)seg * H + h] = f_total;
      } else {
        a.m_next[(int64_t)entry * H + h] = m;
      }
    }
  }
}

// Contributions of an entry's segments -> the state in front of each of them, in place.  Workgroup = (first segment of an
// entry, slice of the elements of S and n; head).  Slices run fastest: with segments there, the one workgroup in
// num_segments that has work would always fall to the same XCD.  A thread owns four consecutive elements; the
// contributions of kAhead segments are loaded together, before the states that replace them are stored.
constexpr int kCombineElements = 1024, kAhead = 8;

template <bool kGates>
__global__ __launch_bounds__(256) void memory_combine_kernel(const MemoryChunkArgs a, int slices) {
  const int seg0 = blockIdx.x / slices, slice = blockIdx.x % slices, h = blockIdx.y;
  const int flags0 = a.segments[4 * seg0 + 3];
  if (!(flags0 & 1) || (flags0 & 4)) return;
  const int slot = a.slot[a.segments[4 * seg0]];
  if (slot < 0) return;
  const int H = a.heads;
  const bool fresh = a.positions[a.segments[4 * seg0 + 1]] == 0;
  const int64_t per_s = (int64_t)a.dim * a.vdim;
  const int64_t at = (int64_t)slice * kCombineElements + 4 * threadIdx.x;
  if (at >= per_s + (kGates ? a.dim : 0)) return;                  // dim and dim * vdim are multiples of four
  const bool in_s = at < per_s;
  const int64_t pitch = in_s ? (int64_t)H * per_s : (int64_t)H * a.dim;         // between segments
  float* ws = in_s ? a.ws_s + h * per_s + at : a.ws_n + (int64_t)h * a.dim + at - per_s;
  float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
  float m = !kGates || fresh ? 0.f : a.m_state[(int64_t)slot * H + h];
  const float log_decay = kGates ? 0.f : a.log_decay[h];
  if (!fresh)
    x = *reinterpret_cast<const float4*>(in_s ? a.s_state + ((int64_t)slot * H + h) * per_s + at
                                              : a.n_state + ((int64_t)slot * H + h) * a.dim + at - per_s);
  for (int base = seg0;; base += kAhead) {
    float4 own[kAhead];
    float f[kAhead], mo[kAhead];
    bool last[kAhead];
#pragma unroll
    for (int j = 0; j < kAhead; ++j) {              // past the entry's last segment: read, not used
      const int seg = min(base + j, a.num_segments - 1);
      own[j] = *reinterpret_cast<const float4*>(ws + seg * pitch);
      f[j] = kGates ? a.ws_f[(int64_t)seg * H + h] : (float)a.segments[4 * seg + 2] * log_decay;
      mo[j] = kGates ? a.ws_m[(int64_t)seg * H + h] : 0.f;
      last[j] = base + j >= a.num_segments - 1 || (a.segments[4 * seg + 3] & 2) != 0;
    }
#pragma unroll
    for (int j = 0; j < kAhead; ++j) {
      *reinterpret_cast<float4*>(ws + (base + j) * pitch) = x;
      if (last[j]) return;
      float m_new = 0.f, keep = 1.f, add = 1.f;
      if constexpr (kGates) {
        m_new = fmaxf(f[j] + m, mo[j]);
        keep = __expf(f[j] + m - m_new);
        add = __expf(mo[j] - m_new);
      } else {
        keep = __expf(f[j]);
      }
      x.x = keep * x.x + add * own[j].x;
      x.y = keep * x.y + add * own[j].y;
      x.z = keep * x.z + add * own[j].z;
      x.w = keep * x.w + add * own[j].w;
      m = m_new;
    }
  }
}
// The maxima in front of the segments: after the kernel above, which still needs the contributions' own.
static __global__ __launch_bounds__(64) void memory_combine_max_kernel(const MemoryChunkArgs a) {
  const int seg0 = blockIdx.x, h = blockIdx.y * 64 + threadIdx.x;
  const int flags0 = a.segments[4 * seg0 + 3];
  if (!(flags0 & 1) || (flags0 & 4) || h >= a.heads) return;
  const int slot = a.slot[a.segments[4 * seg0]];
  if (slot < 0) return;
  float m = a.positions[a.segments[4 * seg0 + 1]] == 0 ? 0.f : a.m_state[(int64_t)slot * a.heads + h];
  for (int seg = seg0; seg < a.num_segments; ++seg) {
    float* p = a.ws_m + (int64_t)seg * a.heads + h;
    const float own = *p;
    *p = m;
    if (a.segments[4 * seg + 3] & 2) break;
    m = fmaxf(a.ws_f[(int64_t)seg * a.heads + h] + m, own);
  }
}

template <int DIMP, int kWaves, bool kGates>
static int launch_chunked(const MemoryChunkArgs& a, bool split, hipStream_t s) {
  const dim3 grid((unsigned)a.num_segments, (unsigned)a.heads, (unsigned)((a.vdim + 32 * kWaves - 1) / (32 * kWaves)));
  const dim3 block(64 * kWaves);
  if (split) {
    memory_chunk_kernel<DIMP, kWaves, true, kGates><<<grid, block, 0, s>>>(a);
    int status = launch_status();
    if (status != 0) return status;
    const int slices = (a.dim * a.vdim + (kGates ? a.dim : 0) + kCombineElements - 1) / kCombineElements;
    if ((int64_t)slices * a.num_segments >= 1 << 24) return MVLLM_ERR_BAD_SHAPE;
    memory_combine_kernel<kGates><<<dim3((unsigned)(slices * a.num_segments), (unsigned)a.heads), dim3(256), 0, s>>>(a, slices);
    if constexpr (kGates)
      memory_combine_max_kernel<<<dim3((unsigned)a.num_segments, (unsigned)((a.heads + 63) / 64)), dim3(64), 0, s>>>(a);
    status = launch_status();
    if (status != 0) return status;
  }
  memory_chunk_kernel<DIMP, kWaves, false, kGates><<<grid, block, 0, s>>>(a);
  return launch_status();
}

template <bool kGates>
static int launch_chunked_sizes(const MemoryChunkArgs& a, bool split, hipStream_t s) {
  if (a.vdim <= 64) {
    if (a.dim <= 64) return launch_chunked<64, 2, kGates>(a, split, s);
    if (a.dim <= 128) return launch_chunked<128, 2, kGates>(a, split, s);
    return launch_chunked<256, 2, kGates>(a, split, s);
  }
  if (a.dim <= 64) return launch_chunked<64, 4, kGates>(a, split, s);
  if (a.dim <= 128) return launch_chunked<128, 4, kGates>(a, split, s);
  return launch_chunked<256, 4, kGates>(a, split, s);
}

}  // namespace mvllm
