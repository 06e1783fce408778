// Mixture of experts: the router's choice, the rows sorted by expert, and the experts' products.
//   moe_route   scores s = sigmoid(z), choice scores s + correction; groups of neighbouring experts by the sum of their two
//               largest choice scores, the best `keep` groups stay open; the `top` largest choice scores of those are chosen,
//               weights s / (sum of the chosen s + 1e-20); or s = softmax(z), the weights s as they are; the last outputs may
//               stand for no expert but for the input itself: their id is -1
//   moe_plan    (token, choice) pairs sorted by expert, and tiles of 128 or 256 sorted rows per expert
//   moe_linear  out[row] = x[row] W_e^T, optionally silu(gate) * up or its clamped form behind it: W_e [2 F, K] with gate and up rows in turns of
//               32, so that both halves of an output are in one lane
// Products, by the number of rows: very few (no plan; a workgroup finds its expert's rows itself, its waves share K), many (bf16: 128 x 128 or 256 x 256
// tiles on the matrix unit over sorted rows), any (fp32, over sorted rows).
#include "prefill_tiles.h"

#pragma clang fp contract(off)

namespace mvllm {

// ---- routing ----
struct RouteArgs {
  int32_t* ids;            // [T, top]
  float* weights;          // [T, top]
  const float* z;          // [T, z_stride] logits
  const float* correction; // [E] or null
  int64_t z_stride;
  int rows, experts, top, groups, keep;
  int identity;            // of the experts: the last ones, whose output is their input
  bool softmax, renormalize;
};

// One token per wave; lane l has experts l, l + 64, ...
template <int NE>
__global__ __launch_bounds__(256) void moe_route_kernel(const RouteArgs a) {
  __shared__ float choice_of[4][64 * NE], group_of[4][64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int row = blockIdx.x * 4 + wave;
  const bool live = row < a.rows;
  const int E = a.experts;
  float s[NE], choice[NE];
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int e = lane + 64 * i;
    s[i] = 0.f;
    choice[i] = -INFINITY;
    if (live && e < E) {
      const float z = a.z[(int64_t)row * a.z_stride + e];
      s[i] = a.softmax ? z : 1.0f / (1.0f + expf(-z));
    }
  }
  if (a.softmax) {
    float most = -INFINITY, sum = 0.f;
#pragma unroll
    for (int i = 0; i < NE; ++i) most = fmaxf(most, lane + 64 * i < E ? s[i] : -INFINITY);
    most = wave_max_in_registers(most);
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      s[i] = lane + 64 * i < E ? expf(s[i] - most) : 0.f;
      sum += s[i];
    }
    sum = four_rows_sum(row16_sum(sum));
#pragma unroll
    for (int i = 0; i < NE; ++i) s[i] /= sum;
  }
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int e = lane + 64 * i;
    if (live && e < E) choice[i] = s[i] + (a.correction ? a.correction[e] : 0.f);
    choice_of[wave][e] = choice[i];
  }
  if (a.groups > 1) {
    const int size = E / a.groups;
    __syncthreads();
    if (lane < a.groups) {
      float first = -INFINITY, second = -INFINITY;
      for (int j = 0; j < size; ++j) {
        const float x = choice_of[wave][lane * size + j];
        second = fmaxf(second, fminf(first, x));
        first = fmaxf(first, x);
      }
      group_of[wave][lane] = size > 1 ? first + second : first;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int e = lane + 64 * i;
      if (e >= E) continue;
      const int g = e / size;
      const float mine = group_of[wave][g];
      int before = 0;
      for (int j = 0; j < a.groups; ++j) {
        const float x = group_of[wave][j];
        before += x > mine || (x == mine && j < g);
      }
      if (before >= a.keep) choice[i] = -INFINITY;
    }
  }
  float my_s = 0.f, sum = 0.f;
  int my_id = 0;
  for (int k = 0; k < a.top; ++k) {
    float mine = choice[0];
#pragma unroll
    for (int i = 1; i < NE; ++i) mine = fmaxf(mine, choice[i]);
    const float best = wave_max_in_registers(mine);
    int id = -1;                                    // the first expert that has it
    float best_s = 0.f;
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const unsigned long long at = __ballot(choice[i] == best);
      if (id < 0 && at != 0ull) {
        const int l = __builtin_amdgcn_readfirstlane(__builtin_ctzll(at));
        id = 64 * i + l;
        best_s = __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(s[i]), l));
        if (lane == l) choice[i] = -INFINITY;
      }
    }
    if (id < 0 || id >= E) id = 0;                  // (nothing left to choose)
    sum += best_s;
    if (lane == k) { my_s = best_s; my_id = id; }
  }
  if (live && lane < a.top) {
    a.ids[(int64_t)row * a.top + lane] = my_id < E - a.identity ? my_id : -1;
    a.weights[(int64_t)row * a.top + lane] = a.renormalize ? my_s / (sum + 1e-20f) : my_s;
  }
}

// ---- pairs sorted by expert ----
constexpr int kPlanPairs = 2048, kMaxExperts = 1024;
constexpr int kLargeTileRows = 384;      // rows per expert from which tiles are large

struct PlanArgs {
  const int32_t* ids;      // [pairs]
  int32_t* hist;           // [blocks, E]
  int32_t* sorted_pair;    // [pairs]: pair at a sorted place
  int32_t* place;          // [pairs]: sorted place of a pair
  int32_t* row_start;      // [E + 1]
  int32_t* tile_expert;    // [max tiles]
  int32_t* tile_row;       // [max tiles]: first sorted row
  int32_t* num_tiles;      // [1]
  int pairs, experts, blocks, tile_rows;
};

__global__ __launch_bounds__(256) void moe_count_kernel(const PlanArgs a) {
  __shared__ int32_t count[kMaxExperts];
  for (int e = threadIdx.x; e < a.experts; e += 256) count[e] = 0;
  __syncthreads();
  const int end = min((int)(blockIdx.x + 1) * kPlanPairs, a.pairs);
  for (int p = blockIdx.x * kPlanPairs + threadIdx.x; p < end; p += 256) {
    const int id = a.ids[p];
    if (id >= 0) atomicAdd(&count[id], 1);
  }
  __syncthreads();
  for (int e = threadIdx.x; e < a.experts; e += 256) a.hist[(int64_t)blockIdx.x * a.experts + e] = count[e];
}

__global__ __launch_bounds__(1024) void moe_place_kernel(const PlanArgs a) {
  __shared__ int32_t total[kMaxExperts + 1], tiles[kMaxExperts + 1], cursor[kMaxExperts];
  const int e = threadIdx.x;
  int n = 0, mine = 0;
  if (a.blocks == 1) {                              // counted here
    cursor[e] = 0;
    __syncthreads();
    for (int p = e; p < a.pairs; p += 1024) {
      const int id = a.ids[p];
      if (id >= 0) atomicAdd(&cursor[id], 1);
    }
    __syncthreads();
    n = cursor[e];
    __syncthreads();
  } else if (e < a.experts)
    for (int b = 0; b < a.blocks; ++b) {
      if (b == (int)blockIdx.x) mine = n;
      n += a.hist[(int64_t)b * a.experts + e];
    }
  // inclusive sums over the experts
  total[e + 1] = n;
  tiles[e + 1] = (n + a.tile_rows - 1) / a.tile_rows;
  if (e == 0) total[0] = tiles[0] = 0;
  __syncthreads();
  for (int o = 1; o < 1024; o <<= 1) {
    const int x = e + 1 > o ? total[e + 1 - o] : 0, y = e + 1 > o ? tiles[e + 1 - o] : 0;
    __syncthreads();
    total[e + 1] += x;
    tiles[e + 1] += y;
    __syncthreads();
  }
  if (e < a.experts) cursor[e] = total[e] + mine;
  __syncthreads();
  const int end = min((int)(blockIdx.x + 1) * kPlanPairs, a.pairs);
  for (int p = blockIdx.x * kPlanPairs + threadIdx.x; p < end; p += 1024) {
    const int id = a.ids[p];
    if (id < 0) {                                   // no expert's: nobody computes or reads it
      a.place[p] = -1;
      continue;
    }
    const int at = atomicAdd(&cursor[id], 1);
    a.sorted_pair[at] = p;
    a.place[p] = at;
  }
  if (blockIdx.x == 0 && e < a.experts) {
    a.row_start[e] = total[e];
    if (e == a.experts - 1) {
      a.row_start[e + 1] = total[e + 1];
      a.num_tiles[0] = tiles[e + 1];
    }
    for (int t = tiles[e]; t < tiles[e + 1]; ++t) {
      a.tile_expert[t] = e;
      a.tile_row[t] = total[e] + (t - tiles[e]) * a.tile_rows;
    }
  }
}

// ---- products ----
struct ExpertLinearArgs {
  void* out;                   // [pairs, out_stride]
  const void* x;               // [*, x_stride]
  const void* w;               // [E, N, K]
  const int32_t* ids;          // [pairs] (few)
  const int32_t* sorted_pair;  // (many, any) plan, see above
  const int32_t* row_start;
  const int32_t* tile_expert;
  const int32_t* tile_row;
  const int32_t* num_tiles;
  int64_t x_stride, out_stride;
  int pairs, experts, N, K;
  int per_token;               // > 0: pair p reads row p / per_token of x; 0: the row of its own (sorted) place
  int max_tiles, n_tiles;
  uint32_t x_bytes;            // (many) what x holds
  float alpha, limit, shift;   // of kClampedGlu
};

enum { kNoGlu = 0, kSiluGlu = 1, kClampedGlu = 2 };

// silu(g) * u, or with g' = min(g, limit) and u' = u within +-limit: g' sigmoid(alpha g') (u' + shift)
template <int kGlu> __device__ __forceinline__ float glu_of(const ExpertLinearArgs& a, float g, float u) {
  if constexpr (kGlu == kClampedGlu) {
    g = fminf(g, a.limit);
    return g * __builtin_amdgcn_rcpf(1.0f + __expf(-a.alpha * g)) * (fminf(fmaxf(u, -a.limit), a.limit) + a.shift);
  }
  return g * __builtin_amdgcn_rcpf(1.0f + __expf(-g)) * u;
}

// few: workgroup = (16 kTiles outputs, expert), its waves share K.  The rows of the expert are found in `ids`; rows are taken
// 16 at a time.
constexpr int kFewPairs = 512;

template <int kWaves, int kGlu, int kTiles>
__global__ __launch_bounds__(64 * kWaves) void moe_linear_few_kernel(const ExpertLinearArgs a) {
  constexpr int NT = kTiles * (kGlu ? 2 : 1);        // tiles of weight rows: with the gate, gate and up of an output tile in turn
  __shared__ uint16_t list[kFewPairs];
  __shared__ int found, count[kWaves];
  __shared__ float4 part[kWaves][NT][64];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4, i16 = lane & 15;
  const int e = blockIdx.y;
  // the expert's pairs, in order: every wave looks through its share of the list, all loads at once
  constexpr int kEach = (kFewPairs + 64 * kWaves - 1) / (64 * kWaves);
  {
    const int share = (a.pairs + 64 * kWaves - 1) / (64 * kWaves) * 64, base = wave * share;
    int32_t id[kEach];
#pragma unroll
    for (int i = 0; i < kEach; ++i) {
      const int p = base + 64 * i + lane;
      id[i] = 64 * i < share && p < a.pairs ? a.ids[p] : -1;
    }
    int n = 0;
#pragma unroll
    for (int i = 0; i < kEach; ++i) n += __popcll(__ballot(id[i] == e));
    if (lane == 0) count[wave] = n;
    __syncthreads();
    int at = 0, all = 0;
#pragma unroll
    for (int i = 0; i < kWaves; ++i) {
      at += i < wave ? count[i] : 0;
      all += count[i];
    }
    if (tid == 0) found = all;
    if (all == 0) return;                           // (the same for every thread)
#pragma unroll
    for (int i = 0; i < kEach; ++i) {
      const bool hit = id[i] == e;
      const unsigned long long hits = __ballot(hit);
      if (hit) list[at + __popcll(hits & ((1ull << lane) - 1))] = (uint16_t)(base + 64 * i + lane);
      at += __popcll(hits);
    }
  }
  __syncthreads();
  const int rows = found;
  const int n0 = blockIdx.x * 16 * kTiles;          // first output of the workgroup
  const bf16_t* w[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    const int out = kGlu ? n0 + 16 * (n / 2) : n0 + 16 * n;
    const int wr = kGlu ? (out >> 5) * 64 + (out & 31) + 32 * (n % 2) : out;
    w[n] = reinterpret_cast<const bf16_t*>(a.w) + ((int64_t)e * a.N + min(wr + i16, a.N - 1)) * a.K;
  }
  for (int r0 = 0; r0 < rows; r0 += 16) {
    const int pair = list[min(r0 + i16, rows - 1)];
    const bf16_t* x = reinterpret_cast<const bf16_t*>(a.x) + (int64_t)(a.per_token ? pair / a.per_token : pair) * a.x_stride;
    v4f acc[NT];
#pragma unroll
    for (int n = 0; n < NT; ++n) acc[n] = v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
    for (int k0 = 64 * wave; k0 < a.K; k0 += 64 * kWaves) {            // a lane's 32 bytes: whole lines per row and wave
      const int k = k0 + 16 * g;
      uint4 xv[2], wv[NT][2];
#pragma unroll
      for (int half = 0; half < 2; ++half) {
#pragma unroll
        for (int n = 0; n < NT; ++n) wv[n][half] = load16_stream(w[n] + k + 8 * half);
        xv[half] = *reinterpret_cast<const uint4*>(x + k + 8 * half);
      }
#pragma unroll
      for (int half = 0; half < 2; ++half)
#pragma unroll
        for (int n = 0; n < NT; ++n) acc[n] = mfma16x16x32<bf16_t>(wv[n][half], xv[half], acc[n]);
    }
    // lane: row i16, outputs 4 g + r
#pragma unroll
    for (int n = 0; n < NT; ++n) part[wave][n][lane] = make_float4(acc[n][0], acc[n][1], acc[n][2], acc[n][3]);
    __syncthreads();
    for (int m = wave; m < kTiles; m += kWaves) {   // output tile
      constexpr int kParts = kGlu ? 2 : 1;
      float z[kParts][4];
#pragma unroll
      for (int n = 0; n < kParts; ++n) {
        z[n][0] = z[n][1] = z[n][2] = z[n][3] = 0.f;
#pragma unroll
        for (int i = 0; i < kWaves; ++i) {
          const float4 p = part[i][m * kParts + n][lane];
          z[n][0] += p.x; z[n][1] += p.y; z[n][2] += p.z; z[n][3] += p.w;
        }
      }
      float o[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] = kGlu ? glu_of<kGlu>(a, z[0][r], z[kParts - 1][r]) : z[0][r];
      const int col = n0 + 16 * m + 4 * g;
      bf16_t* out = reinterpret_cast<bf16_t*>(a.out) + (int64_t)pair * a.out_stride + col;
      if (r0 + i16 < rows && col < (kGlu ? a.N / 2 : a.N)) *reinterpret_cast<uint2*>(out) = make_uint2(pack2<bf16_t>(o[0], o[1]), pack2<bf16_t>(o[2], o[3]));
    }
    __syncthreads();
  }
}

// any: workgroup = (16 outputs, expert, every gridDim.z-th 16 sorted rows), one dot product (two with the gate) per thread.
template <typename T, int kGlu>
__global__ __launch_bounds__(256) void moe_linear_any_kernel(const ExpertLinearArgs a) {
  constexpr int kStep = 64, NT = kGlu ? 2 : 1;
  __shared__ float xs[16][kStep + 1], ws[NT][16][kStep + 1];
  const int tid = threadIdx.x, r = tid >> 4, c = tid & 15, e = blockIdx.y, n0 = blockIdx.x * 16;
  const int first = a.row_start[e], last = a.row_start[e + 1];
  for (int base = first + 16 * blockIdx.z; base < last; base += 16 * gridDim.z) {
    float acc[NT];
#pragma unroll
    for (int n = 0; n < NT; ++n) acc[n] = 0.f;
    for (int k0 = 0; k0 < a.K; k0 += kStep) {
      for (int i = tid; i < 16 * kStep; i += 256) {
        const int rr = i / kStep, k = k0 + i % kStep, at = base + rr;
        float xv = 0.f;
        if (at < last && k < a.K)
          xv = to_float(reinterpret_cast<const T*>(a.x)[(int64_t)(a.per_token ? a.sorted_pair[at] / a.per_token : at) * a.x_stride + k]);
        xs[rr][i % kStep] = xv;
#pragma unroll
        for (int n = 0; n < NT; ++n) {
          const int wr = kGlu ? ((n0 + rr) >> 5) * 64 + ((n0 + rr) & 31) + 32 * n : n0 + rr;
          ws[n][rr][i % kStep] = wr < a.N && k < a.K ? to_float(reinterpret_cast<const T*>(a.w)[((int64_t)e * a.N + wr) * a.K + k]) : 0.f;
        }
      }
      __syncthreads();
#pragma unroll 16
      for (int k = 0; k < kStep; ++k)
#pragma unroll
        for (int n = 0; n < NT; ++n) acc[n] = fmaf(xs[r][k], ws[n][c][k], acc[n]);
      __syncthreads();
    }
    if (base + r < last) {
      float o = acc[0];
      if constexpr (kGlu == kSiluGlu) o = acc[0] / (1.0f + expf(-acc[0])) * acc[NT - 1];
      if constexpr (kGlu == kClampedGlu) {
        const float z = fminf(acc[0], a.limit);
        o = z / (1.0f + expf(-a.alpha * z)) * (fminf(fmaxf(acc[NT - 1], -a.limit), a.limit) + a.shift);
      }
      reinterpret_cast<T*>(a.out)[(int64_t)(base + r) * a.out_stride + n0 + c] = from_float<T>(o);
    }
  }
}

// many: 128 sorted rows x 128 weight rows per workgroup, four waves of 64 x 64 on v_mfma_f32_32x32x16_bf16.  Weights are the
// row operand and x the column operand, so that a lane ends with runs of four outputs of one row.  Steps of 64 along K, two
// buffers in LDS that the copies of the next step fill during this one; a row's eight 16-byte chunks trade places by half
// the row's number.  Consecutive workgroups of an XCD go through four row tiles for every weight tile.
template <int kGlu>
__global__ __launch_bounds__(256, 2) void moe_linear_many_kernel(const ExpertLinearArgs a) {
  constexpr int kTile = 128, kK = 64, kStage = kTile * kK * 2;       // bytes of one operand's step
  constexpr int kTogether = 4;
  __shared__ __attribute__((aligned(16))) char lds[4 * kStage];      // [buffer][weights, x]
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), l32 = lane & 31, hi = lane >> 5;
  // ---- which tile ----
  const int total = a.num_tiles[0], per = (total + 7) / 8;
  const int xcd = blockIdx.x & 7, j = blockIdx.x >> 3;
  const int group = j / (kTogether * a.n_tiles), in_group = j % (kTogether * a.n_tiles);
  const int local = group * kTogether + in_group % kTogether, tile = xcd * per + local, n_tile = in_group / kTogether;
  if (local >= per || tile >= total) return;
  const int e = a.tile_expert[tile], row0 = a.tile_row[tile], row_end = min(row0 + kTile, a.row_start[e + 1]);
  const int n0 = n_tile * kTile;

  // ---- copies: four chunks of either operand per thread and step ----
  const v4i w_rows = make_rsrc(reinterpret_cast<const char*>(a.w) + (int64_t)e * a.N * a.K * 2, (uint32_t)((int64_t)a.N * a.K * 2));
  const v4i x_rows = make_rsrc(reinterpret_cast<const char*>(a.x), a.x_bytes);
  uint32_t from_w[4], from_x[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int c = 256 * i + tid, r = c >> 3, p = (c & 7) ^ ((r >> 1) & 7);
    from_w[i] = (uint32_t)(min(n0 + r, a.N - 1) * a.K + 8 * p) * 2u;
    const int at = min(row0 + r, row_end - 1);
    const uint32_t xr = (uint32_t)(a.per_token ? a.sorted_pair[at] / a.per_token : at);
    from_x[i] = (xr * (uint32_t)a.x_stride + 8u * p) * 2u;
  }
  auto copy = [&](int buffer) __attribute__((always_inline)) {
    const uint32_t base = lds_address(lds) + buffer * 2 * kStage + 1024 * wave;
    static_for<4>([&](auto I) {
      constexpr int i = decltype(I)::value;
      dma16_to_lds<4096 * i>(w_rows, from_w[i], base);
      dma16_to_lds<kStage + 4096 * i>(x_rows, from_x[i], base);
      from_w[i] += 2 * kK;
      from_x[i] += 2 * kK;
    });
  };
  const int wn = wave & 1, wm = wave >> 1;          // the wave's half of the weight rows and of the rows
  // places of this lane's fragments: row l32 of a 32-row block, chunk 2 st + hi
  const int sw = (l32 >> 1) & 7;
  const char* frag = lds + l32 * 128;
  v16f acc[2][2];
#pragma unroll
  for (int n = 0; n < 2; ++n)
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[n][m][r] = 0.f;

  copy(0);
  const int steps = a.K / kK;
  for (int step = 0; step < steps; ++step) {
    const int buffer = step & 1;
    dma_wait_all();
    __syncthreads();                                // this step's operands are there, the other buffer is free
    if (step + 1 < steps) copy(buffer ^ 1);
    const char* wb = frag + buffer * 2 * kStage + wn * 64 * 128;
    const char* xb = frag + buffer * 2 * kStage + kStage + wm * 64 * 128;
#pragma unroll
    for (int st = 0; st < 4; ++st) {
      const int p = ((2 * st + hi) ^ sw) << 4;
      uint4 wf[2], xf[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        wf[i] = *reinterpret_cast<const uint4*>(wb + i * 32 * 128 + p);
        xf[i] = *reinterpret_cast<const uint4*>(xb + i * 32 * 128 + p);
      }
#pragma unroll
      for (int n = 0; n < 2; ++n)
#pragma unroll
        for (int m = 0; m < 2; ++m) acc[n][m] = mfma32x32x16<bf16_t>(wf[n], xf[m], acc[n][m]);
    }
  }
  // ---- lane: row l32 of a block, weight rows 8 (r / 4) + 4 hi + r % 4 ----
#pragma unroll
  for (int m = 0; m < 2; ++m) {
    const int row = row0 + wm * 64 + 32 * m + l32;
    if (row >= row_end) continue;
    bf16_t* out = reinterpret_cast<bf16_t*>(a.out) + (int64_t)row * a.out_stride;
#pragma unroll
    for (int r = 0; r < 16; r += 4) {
      if constexpr (kGlu) {
        const int col = (n0 + wn * 64) / 2 + 2 * r + 4 * hi;
        float o[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) o[i] = glu_of<kGlu>(a, acc[0][m][r + i], acc[1][m][r + i]);
        if (2 * col < a.N) *reinterpret_cast<uint2*>(out + col) = make_uint2(pack2<bf16_t>(o[0], o[1]), pack2<bf16_t>(o[2], o[3]));
      } else {
#pragma unroll
        for (int n = 0; n < 2; ++n) {
          const int col = n0 + wn * 64 + 32 * n + 2 * r + 4 * hi;
          if (col < a.N)
            *reinterpret_cast<uint2*>(out + col) = make_uint2(pack2<bf16_t>(acc[n][m][r], acc[n][m][r + 1]), pack2<bf16_t>(acc[n][m][r + 2], acc[n][m][r + 3]));
        }
      }
    }
  }
}

// many, large tiles: 256 sorted rows x 256 weight rows, four waves of 128 x 128 (a wave's accumulators fill half its SIMD's
// registers; per flop it reads half as much of LDS as with 64 x 64).  The operands of a 16-wide step are read during the
// products of the one before; a step's last products hide the barrier, after which the next step's operands are there and
// more copies start: x, which other workgroups of the XCD read too, one step ahead in two buffers, the weights, which come
// from memory, two steps ahead in three.  Together they fill the LDS.
template <int kGlu>
__global__ __launch_bounds__(256, 1) void moe_linear_large_kernel(const ExpertLinearArgs a) {
  constexpr int kTile = 256, kK = 64, kStage = kTile * kK * 2;       // bytes of one operand's step
  constexpr int kTogether = 4;
  __shared__ __attribute__((aligned(16))) char lds[5 * kStage];      // weights three times, x twice
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), l32 = lane & 31, hi = lane >> 5;
  const int total = a.num_tiles[0], per = (total + 7) / 8;
  const int xcd = blockIdx.x & 7, j = blockIdx.x >> 3;
  const int group = j / (kTogether * a.n_tiles), in_group = j % (kTogether * a.n_tiles);
  const int local = group * kTogether + in_group % kTogether, tile = xcd * per + local, n_tile = in_group / kTogether;
  if (local >= per || tile >= total) return;
  const int e = a.tile_expert[tile], row0 = a.tile_row[tile], row_end = min(row0 + kTile, a.row_start[e + 1]);
  const int n0 = n_tile * kTile;

  const v4i w_rows = make_rsrc(reinterpret_cast<const char*>(a.w) + (int64_t)e * a.N * a.K * 2, (uint32_t)((int64_t)a.N * a.K * 2));
  const v4i x_rows = make_rsrc(reinterpret_cast<const char*>(a.x), a.x_bytes);
  uint32_t from_w[8], from_x[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const int c = 256 * i + tid, r = c >> 3, p = (c & 7) ^ ((r >> 1) & 7);
    from_w[i] = (uint32_t)(min(n0 + r, a.N - 1) * a.K + 8 * p) * 2u;
    const int at = min(row0 + r, row_end - 1);
    const uint32_t xr = (uint32_t)(a.per_token ? a.sorted_pair[at] / a.per_token : at);
    from_x[i] = (xr * (uint32_t)a.x_stride + 8u * p) * 2u;
  }
  constexpr int kX = 3 * kStage;                    // where x begins
  const uint32_t lds_wave = lds_address(lds) + 1024 * wave;
  const int steps = a.K / kK;
  // copy i of eight of a step's operand; past the last step nothing is read (the buffer is not used again)
  auto copy_w = [&](auto I, int step, uint32_t buffer) __attribute__((always_inline)) {
    v4i rows = w_rows;
    rows[2] = step < steps ? rows[2] : 0;
    dma16_to_lds_at<4096 * decltype(I)::value>(rows, from_w[decltype(I)::value], (uint32_t)step * (2 * kK), lds_wave + buffer);
  };
  auto copy_x = [&](auto I, int step) __attribute__((always_inline)) {
    v4i rows = x_rows;
    rows[2] = step < steps ? rows[2] : 0;
    dma16_to_lds_at<4096 * decltype(I)::value>(rows, from_x[decltype(I)::value], (uint32_t)step * (2 * kK), lds_wave + kX + (step & 1) * kStage);
  };
  const int wn = wave & 1, wm = wave >> 1;
  const int sw = (l32 >> 1) & 7;
  const char* frag = lds + l32 * 128;
  v16f acc[4][4];
#pragma unroll
  for (int n = 0; n < 4; ++n)
#pragma unroll
    for (int m = 0; m < 4; ++m)
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[n][m][r] = 0.f;
  uint4 wf[2][4], xf[2][4];
  // where this lane's operands of the four 16-wide steps lie in a buffer
  uint32_t place[4];
#pragma unroll
  for (int st = 0; st < 4; ++st) place[st] = ((2 * st + hi) ^ sw) << 4;
  const char* w_frag = frag + wn * (128 * 128);
  const char* x_frag = frag + wm * (128 * 128) + kX;
  // The products of a 16-wide step one by one; after each of them one of the next step's reads (every kEvery-th from product
  // kFirst on, those that are needed first come first) and whatever `also` does: the matrix unit must not wait for a queue of
  // reads or copies.
  auto products = [&](auto SET, auto FIRST, auto EVERY, const char* wb, const char* xb, auto&& also) __attribute__((always_inline)) {
    constexpr int set = decltype(SET)::value, next = set ^ 1, kFirst = decltype(FIRST)::value, kEvery = decltype(EVERY)::value;
    static_for<16>([&](auto I) {
      constexpr int i = decltype(I)::value;
      acc[i / 4][i % 4] = mfma32x32x16<bf16_t>(wf[set][i / 4], xf[set][i % 4], acc[i / 4][i % 4]);
      also(I);
      if constexpr (i >= kFirst && (i - kFirst) % kEvery == 0 && (i - kFirst) / kEvery < 8) {
        constexpr int j = (i - kFirst) / kEvery;
        if constexpr (j >= 1 && j <= 4) xf[next][j - 1] = *reinterpret_cast<const uint4*>(xb + (j - 1) * 32 * 128);
        else wf[next][j == 0 ? 0 : j - 4] = *reinterpret_cast<const uint4*>(wb + (j == 0 ? 0 : j - 4) * 32 * 128);
      }
      __builtin_amdgcn_sched_barrier(0);
    });
  };
  constexpr std::integral_constant<int, 0> c0{};
  constexpr std::integral_constant<int, 1> c1{};
  constexpr std::integral_constant<int, 2> c2{};
  constexpr std::integral_constant<int, 4> c4{};
  auto nothing = [](auto) {};

  static_for<8>([&](auto I) {
    copy_w(I, 0, 0);
    copy_x(I, 0);
    copy_w(I, 1, kStage);
  });
  dma_wait_all();
  __syncthreads();
  static_for<8>([&](auto I) { copy_x(I, 1); });
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    wf[0][i] = *reinterpret_cast<const uint4*>(w_frag + place[0] + i * 32 * 128);
    xf[0][i] = *reinterpret_cast<const uint4*>(x_frag + place[0] + i * 32 * 128);
  }
  uint32_t w_at = 0;                                // the weights' buffer of this step, in bytes
  for (int step = 0; step < steps; ++step) {
    const uint32_t w_next = w_at == 2 * kStage ? 0 : w_at + kStage, w_free = w_at == 0 ? 2 * kStage : w_at - kStage;
    const char* wb = w_frag + w_at;
    const char* xb = x_frag + (step & 1) * kStage;
    // the weights two steps ahead, into the buffer that the step before this one has left
    products(c0, c1, c2, wb + place[1], xb + place[1], [&](auto I) {
      constexpr int i = decltype(I)::value;
      if constexpr (i % 2 == 0) copy_w(std::integral_constant<int, i / 2>{}, step + 2, w_free);
    });
    products(c1, c1, c2, wb + place[2], xb + place[2], nothing);
    products(c0, c1, c2, wb + place[3], xb + place[3], nothing);
    // the next step's operands have to be there before its first reads, and this step's have been read: then x two steps
    // ahead follows into its buffer.  What may be in flight until then are the eight copies of weights from above.
    products(c1, c4, c1, w_frag + w_next + place[0], x_frag + ((step & 1) ^ 1) * kStage + place[0], [&](auto I) {
      constexpr int i = decltype(I)::value;
      if constexpr (i == 3) {
        dma_wait_but<8>();
        workgroup_barrier();
      }
      if constexpr (i >= 8) copy_x(std::integral_constant<int, i - 8>{}, step + 2);
    });
    w_at = w_next;
  }
  dma_wait_all();                                   // (copies past the last step)
  // ---- lane: row l32 of a block, weight rows 8 (r / 4) + 4 hi + r % 4; halves of the wave trade runs of four, so that a lane
  // stores eight outputs in a row ----
#pragma unroll
  for (int m = 0; m < 4; ++m) {
    const int row = row0 + wm * 128 + 32 * m + l32;
    bf16_t* out = reinterpret_cast<bf16_t*>(a.out) + (int64_t)min(row, row_end - 1) * a.out_stride;
#pragma unroll
    for (int n = 0; n < (kGlu ? 2 : 4); ++n) {
#pragma unroll
      for (int r = 0; r < 16; r += 8) {
        float o[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          if constexpr (kGlu) o[i] = glu_of<kGlu>(a, acc[2 * n][m][r + i], acc[2 * n + 1][m][r + i]);
          else o[i] = acc[n][m][r + i];
        }
        const auto x = __builtin_amdgcn_permlane32_swap(pack2<bf16_t>(o[0], o[1]), pack2<bf16_t>(o[4], o[5]), false, false);
        const auto y = __builtin_amdgcn_permlane32_swap(pack2<bf16_t>(o[2], o[3]), pack2<bf16_t>(o[6], o[7]), false, false);
        const int col = (kGlu ? (n0 + wn * 128) / 2 : n0 + wn * 128) + 32 * n + 2 * r + 8 * hi;
        if (row < row_end && col < (kGlu ? a.N / 2 : a.N)) *reinterpret_cast<uint4*>(out + col) = make_uint4(x[0], y[0], x[1], y[1]);
      }
    }
  }
}

// Rows of a tile: large ones where experts have enough rows on average to fill them.
static int tile_rows(int64_t pairs, int experts) { return pairs >= kLargeTileRows * (int64_t)experts ? 256 : 128; }
static int64_t max_tiles(int64_t pairs, int experts) { return (pairs + tile_rows(pairs, experts) - 1) / tile_rows(pairs, experts) + experts; }
static int plan_blocks(int64_t pairs) { return (int)((pairs + kPlanPairs - 1) / kPlanPairs); }

}  // namespace mvllm

using namespace mvllm;

static int route(RouteArgs a, int64_t rows, void* stream) {
  if (rows < 0 || a.experts <= 0 || a.top <= 0 || a.top > a.experts || a.groups <= 0 || a.experts % a.groups != 0 || a.keep <= 0 ||
      a.keep > a.groups || a.z_stride < a.experts || (int64_t)a.keep * (a.experts / a.groups) < a.top || a.identity < 0 || a.identity > a.experts)
    return MVLLM_ERR_BAD_SHAPE;
  if (a.experts > kMaxExperts || a.top > 64 || a.groups > 64 || rows > (1 << 28)) return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0) return MVLLM_OK;
  if (!a.ids || !a.weights || !a.z) return MVLLM_ERR_NULL_POINTER;
  a.rows = (int)rows;
  const dim3 grid((unsigned)((rows + 3) / 4)), block(256);
  hipStream_t s = (hipStream_t)stream;
  if (a.experts <= 64) moe_route_kernel<1><<<grid, block, 0, s>>>(a);
  else if (a.experts <= 128) moe_route_kernel<2><<<grid, block, 0, s>>>(a);
  else if (a.experts <= 256) moe_route_kernel<4><<<grid, block, 0, s>>>(a);
  else moe_route_kernel<16><<<grid, block, 0, s>>>(a);
  return launch_status();
}

extern "C" int mvllm_moe_route(int32_t* ids, float* weights, const float* logits, int64_t logit_row_stride,
                               const float* correction, int64_t rows, int experts, int top, int groups, int keep,
                               void* stream) {
  RouteArgs a = {};
  a.ids = ids; a.weights = weights; a.z = logits; a.correction = correction; a.z_stride = logit_row_stride;
  a.experts = experts; a.top = top; a.groups = groups; a.keep = keep; a.renormalize = true;
  return route(a, rows, stream);
}

extern "C" int mvllm_moe_route_softmax(int32_t* ids, float* weights, const float* logits, int64_t logit_row_stride,
                                       const float* correction, int64_t rows, int experts, int identity, int top,
                                       int renormalize, void* stream) {
  if (experts < 0 || identity < 0 || experts > kMaxExperts || identity > kMaxExperts) return MVLLM_ERR_BAD_SHAPE;
  RouteArgs a = {};
  a.ids = ids; a.weights = weights; a.z = logits; a.correction = correction; a.z_stride = logit_row_stride;
  a.experts = experts + identity; a.identity = identity; a.top = top; a.groups = 1; a.keep = 1; a.softmax = true;
  a.renormalize = renormalize != 0;
  return route(a, rows, stream);
}

extern "C" size_t mvllm_moe_plan_bytes(int64_t pairs, int experts) {
  if (pairs <= 0 || experts <= 0) return 0;
  return (size_t)(2 * pairs + experts + 1 + 2 * max_tiles(pairs, experts) + 1 + (int64_t)plan_blocks(pairs) * experts + 4) * sizeof(int32_t);
}

// the parts of a plan, in order
static PlanArgs plan_parts_of(void* plan, const int32_t* ids, int64_t pairs, int experts) {
  PlanArgs a;
  a.ids = ids;
  a.place = reinterpret_cast<int32_t*>(plan);
  a.sorted_pair = a.place + pairs;
  a.row_start = a.sorted_pair + pairs;
  a.tile_expert = a.row_start + experts + 1;
  a.tile_row = a.tile_expert + max_tiles(pairs, experts);
  a.num_tiles = a.tile_row + max_tiles(pairs, experts);
  a.hist = a.num_tiles + 1;
  a.pairs = (int)pairs; a.experts = experts; a.blocks = plan_blocks(pairs);
  a.tile_rows = tile_rows(pairs, experts);
  return a;
}

extern "C" int mvllm_moe_plan(void* plan, size_t plan_bytes, const int32_t* ids, int64_t pairs, int experts, void* stream) {
  if (pairs < 0 || experts <= 0) return MVLLM_ERR_BAD_SHAPE;
  if (experts > kMaxExperts || pairs > (1 << 30)) return MVLLM_ERR_UNSUPPORTED;
  if (pairs == 0) return MVLLM_OK;
  if (!plan || !ids) return MVLLM_ERR_NULL_POINTER;
  if (plan_bytes < mvllm_moe_plan_bytes(pairs, experts)) return MVLLM_ERR_WORKSPACE;
  const PlanArgs a = plan_parts_of(plan, ids, pairs, experts);
  hipStream_t s = (hipStream_t)stream;
  if (a.blocks > 1) moe_count_kernel<<<dim3((unsigned)a.blocks), dim3(256), 0, s>>>(a);
  moe_place_kernel<<<dim3((unsigned)a.blocks), dim3(1024), 0, s>>>(a);
  return launch_status();
}

// f(a kGlu as a constant)
template <typename F> static void with_glu(int glu, F f) {
  if (glu == kClampedGlu) f(std::integral_constant<int, kClampedGlu>{});
  else if (glu == kSiluGlu) f(std::integral_constant<int, kSiluGlu>{});
  else f(std::integral_constant<int, kNoGlu>{});
}

static int expert_linear(void* out, int64_t out_row_stride, const void* x, int64_t x_row_stride, const void* w,
                         const int32_t* ids, void* plan, int64_t pairs, int experts, int N, int K, int per_token,
                         int glu, float alpha, float limit, float shift, int dtype, void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (pairs < 0 || experts <= 0 || N <= 0 || K <= 0 || per_token < 0 || x_row_stride < K || out_row_stride < (glu ? N / 2 : N)) return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || experts > kMaxExperts || pairs > (1 << 30) || K % 64 != 0 || N % (glu ? 64 : 16) != 0 || x_row_stride % 8 != 0 ||
      out_row_stride % 4 != 0)
    return MVLLM_ERR_UNSUPPORTED;
  if (pairs == 0) return MVLLM_OK;
  if (!out || !x || !w || (!plan && !ids)) return MVLLM_ERR_NULL_POINTER;
  if (!aligned16(out) || !aligned16(x) || !aligned16(w)) return MVLLM_ERR_MISALIGNED;
  if (!plan && (dtype != MVLLM_BF16 || pairs > kFewPairs)) return MVLLM_ERR_UNSUPPORTED;
  ExpertLinearArgs a = {};
  a.out = out; a.x = x; a.w = w; a.ids = ids; a.x_stride = x_row_stride; a.out_stride = out_row_stride; a.pairs = (int)pairs;
  a.experts = experts; a.N = N; a.K = K; a.per_token = per_token; a.alpha = alpha; a.limit = limit; a.shift = shift;
  hipStream_t s = (hipStream_t)stream;
  const int outputs = glu ? N / 2 : N;
  if (!plan) {
    const unsigned n32 = (unsigned)((outputs + 31) / 32), n64 = (unsigned)((outputs + 63) / 64), n_experts = (unsigned)experts;
    with_glu(glu, [&](auto G) {
      constexpr int kGlu = decltype(G)::value, kTiles = kGlu ? 2 : 4;
      const dim3 grid(kGlu ? n32 : n64, n_experts);
      if (K >= 2048) moe_linear_few_kernel<8, kGlu, kTiles><<<grid, dim3(512), 0, s>>>(a);
      else moe_linear_few_kernel<4, kGlu, kTiles><<<grid, dim3(256), 0, s>>>(a);
    });
    return launch_status();
  }
  const PlanArgs p = plan_parts_of(plan, ids, pairs, experts);
  a.sorted_pair = p.sorted_pair; a.row_start = p.row_start; a.tile_expert = p.tile_expert; a.tile_row = p.tile_row;
  a.num_tiles = p.num_tiles;
  if (dtype == MVLLM_BF16) {
    a.max_tiles = (int)max_tiles(pairs, experts);
    a.n_tiles = (N + p.tile_rows - 1) / p.tile_rows;
    if (p.tile_rows == 256 && out_row_stride % 8 != 0) return MVLLM_ERR_UNSUPPORTED;
    const int64_t x_rows = per_token ? (pairs + per_token - 1) / per_token : pairs, x_bytes = ((x_rows - 1) * x_row_stride + K) * 2;
    if (x_bytes >= (int64_t)1 << 32 || (int64_t)N * K * 2 >= (int64_t)1 << 31) return MVLLM_ERR_UNSUPPORTED;
    a.x_bytes = (uint32_t)x_bytes;
    const int64_t per = (a.max_tiles + 7) / 8, groups = (per + 3) / 4, blocks = 8 * groups * 4 * a.n_tiles;
    if (blocks > 0x7fffffff) return MVLLM_ERR_BAD_SHAPE;
    const bool large = p.tile_rows == 256;
    with_glu(glu, [&](auto G) {
      constexpr int kGlu = decltype(G)::value;
      if (large) moe_linear_large_kernel<kGlu><<<dim3((unsigned)blocks), dim3(256), 0, s>>>(a);
      else moe_linear_many_kernel<kGlu><<<dim3((unsigned)blocks), dim3(256), 0, s>>>(a);
    });
  } else {
    int64_t z = pairs / (16 * (int64_t)experts) + 1;
    const dim3 grid((unsigned)(outputs / 16), (unsigned)experts, (unsigned)(z > 64 ? 64 : z));
    with_glu(glu, [&](auto G) { moe_linear_any_kernel<float, decltype(G)::value><<<grid, dim3(256), 0, s>>>(a); });
  }
  return launch_status();
}

extern "C" int mvllm_moe_linear(void* out, int64_t out_row_stride, const void* x, int64_t x_row_stride, const void* w,
                                const int32_t* ids, void* plan, int64_t pairs, int experts, int N, int K, int per_token,
                                int glu, int dtype, void* stream) {
  return expert_linear(out, out_row_stride, x, x_row_stride, w, ids, plan, pairs, experts, N, K, per_token, glu ? kSiluGlu : kNoGlu,
                       0.f, 0.f, 0.f, dtype, stream);
}

extern "C" int mvllm_moe_linear_clamped(void* out, int64_t out_row_stride, const void* x, int64_t x_row_stride, const void* w,
                                        const int32_t* ids, void* plan, int64_t pairs, int experts, int N, int K,
                                        int per_token, float alpha, float limit, float shift, int dtype, void* stream) {
  return expert_linear(out, out_row_stride, x, x_row_stride, w, ids, plan, pairs, experts, N, K, per_token, kClampedGlu, alpha, limit,
                       shift, dtype, stream);
}
