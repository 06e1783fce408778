// What stands between two sublayers of a decoder with norms on both sides of a sublayer and a short causal convolution in
// front of it, in one launch: the norm of the last sublayer's output, its addition to the fp32 residual stream, the norm
// in front of the next sublayer and the convolution over time of what that norm delivers.
//     x' = x + rms(y) * post          (y null: x' = x; x may come from the embedding table)
//     h  = rms(x') * pre
//     out = h + sum_j conv[j] * h_(t - taps + 1 + j)     (no conv: out = h)
// Norm gains are one number for all channels (stride 0) or one per channel (stride 1).  The convolution's inputs before
// an entry's first row come from the sequence's state (its last taps - 1 values of h, fp32), zeros before position 0.
//
// A workgroup walks `rows_per_wg` consecutive rows, all channels of a row spread over its threads, so that the window of
// the convolution lives in registers and every element is read once.  The taps - 1 rows in front of its first row are
// recomputed (not stored).  Rows are taken kBatch at a time (one channel chunk per thread; wide rows one at a time): their
// loads are issued together and their two sums of squares are reduced together.
// The state is read by an entry's first row and written by its last one; when those belong to different workgroups the
// caller gives the entry two banks (conv_in != conv_out).
#include "row_sums.h"

#pragma clang fp contract(off)

namespace mvllm {

struct NormConvArgs {
  void* out;               // [T, W] element type
  float* x_out;            // [T, W] or null
  const float* x;          // [T, W], or null with `embed`
  const void* embed;       // [vocab, W] element type, or null
  const int64_t* tokens;   // [T], with `embed`
  const void* y;           // [T, W] element type, or null
  const float* post;       // gain of y's norm
  const float* pre;        // gain of the norm in front
  const float* conv;       // [taps, W] or null
  float* state;            // [banks, taps - 1, W]
  const int32_t* cu;       // [entries + 1] rows of the entries
  const int32_t* row_entry;   // [T]
  const int32_t* bank_in;     // [entries]
  const int32_t* bank_out;    // [entries]
  const int64_t* positions;   // [T]
  int64_t vocab;
  float eps;
  int rows;
  int width;
  int post_stride, pre_stride;
  int rows_per_wg;
};

constexpr int kRowsTogether = 4;     // rows reduced together

// NC chunks of VEC channels per thread.
template <typename T, int TAPS, int VEC, int NC>
__global__ __launch_bounds__(kMaxThreads) void norm_conv_kernel(const NormConvArgs a) {
  constexpr int C = VEC * NC;
  constexpr int kHist = TAPS > 1 ? TAPS - 1 : 1;
  constexpr int kBatch = NC == 1 ? kRowsTogether : 1;
  constexpr bool kKeepConv = NC == 1;       // taps and gains in registers; wide rows read them again for every row
  __shared__ __attribute__((aligned(16))) float lds[2 * (kMaxThreads / 16) * kRowsTogether];
  int flip = 0;
  const int waves = blockDim.x >> 6;
  const int W = a.width;
  const int first = blockIdx.x * a.rows_per_wg;
  const int last = min(first + a.rows_per_wg, a.rows);       // one past
  const T* y = reinterpret_cast<const T*>(a.y);
  const T* embed = reinterpret_cast<const T*>(a.embed);
  T* out = reinterpret_cast<T*>(a.out);
  const float inv_w = 1.0f / (float)W;
  int chan[NC];
  bool has[NC];
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    chan[c] = (threadIdx.x + c * blockDim.x) * VEC;
    has[c] = chan[c] < W;
  }
  auto post_at = [&](int c) __attribute__((always_inline)) { return has[c / VEC] && a.y ? a.post[(chan[c / VEC] + c % VEC) * a.post_stride] : 0.f; };
  auto pre_at = [&](int c) __attribute__((always_inline)) { return has[c / VEC] ? a.pre[(chan[c / VEC] + c % VEC) * a.pre_stride] : 0.f; };
  auto conv_at = [&](int j, int c) __attribute__((always_inline)) {
    return has[c / VEC] && a.conv ? a.conv[(int64_t)j * W + chan[c / VEC] + c % VEC] : 0.f;
  };
  constexpr int K = kKeepConv ? C : 1;
  float conv[TAPS][K], post[K], pre[K], hist[kHist][C];
#pragma unroll
  for (int j = 0; j < kHist; ++j)
#pragma unroll
    for (int c = 0; c < C; ++c) hist[j][c] = 0.f;
  if constexpr (kKeepConv) {
#pragma unroll
    for (int c = 0; c < C; ++c) {
      post[c] = post_at(c);
      pre[c] = pre_at(c);
#pragma unroll
      for (int j = 0; j < TAPS; ++j) conv[j][c] = conv_at(j, c);
    }
  }
  // rows in front of the first one that its window reaches into (inside the same entry)
  int start = first;
  if (TAPS > 1 && a.conv) start = first - min(TAPS - 1, first - a.cu[a.row_entry[first]]);

  for (int base = start; base < last; base += kBatch) {
    const int n = min(kBatch, last - base);
    float x[kBatch][C], yv[kBatch][C], sums[kBatch];
#pragma unroll
    for (int r = 0; r < kBatch; ++r) {
      const int64_t row = base + r;
      const T* erow = nullptr;
      if (r < n && embed) {
        const int64_t tok = a.tokens[row];
        erow = embed + (tok < 0 ? 0 : tok >= a.vocab ? a.vocab - 1 : tok) * W;
      }
#pragma unroll
      for (int c = 0; c < NC; ++c) {
        if (r < n && has[c]) {
          if (embed) Chunk<T, VEC>::load(erow + chan[c], &x[r][c * VEC]);
          else Chunk<float, VEC>::load(a.x + row * W + chan[c], &x[r][c * VEC]);
          if (y) Chunk<T, VEC>::load(y + row * W + chan[c], &yv[r][c * VEC]);
        } else {
#pragma unroll
          for (int e = 0; e < VEC; ++e) x[r][c * VEC + e] = yv[r][c * VEC + e] = 0.f;
        }
      }
    }
    if (y) {
#pragma unroll
      for (int r = 0; r < kBatch; ++r) {
        sums[r] = 0.f;
#pragma unroll
        for (int c = 0; c < C; ++c) sums[r] = fmaf(yv[r][c], yv[r][c], sums[r]);
      }
      block_sums<kBatch>(sums, lds, waves, flip);
#pragma unroll
      for (int r = 0; r < kBatch; ++r) {
        const float d = sqrtf(sums[r] * inv_w + a.eps);
        const float s = 1.0f / d;
#pragma unroll
        for (int c = 0; c < C; ++c) x[r][c] += yv[r][c] * s * (kKeepConv ? post[kKeepConv ? c : 0] : post_at(c));
      }
    }
#pragma unroll
    for (int r = 0; r < kBatch; ++r) {
      sums[r] = 0.f;
#pragma unroll
      for (int c = 0; c < C; ++c) sums[r] = fmaf(x[r][c], x[r][c], sums[r]);
    }
    block_sums<kBatch>(sums, lds, waves, flip);
#pragma unroll
    for (int r = 0; r < kBatch; ++r) {
      if (r >= n) break;
      const int row = base + r;
      const bool mine = row >= first;
      const float s = 1.0f / sqrtf(sums[r] * inv_w + a.eps);
      float h[C], o[C];
#pragma unroll
      for (int c = 0; c < C; ++c) o[c] = h[c] = x[r][c] * s * (kKeepConv ? pre[kKeepConv ? c : 0] : pre_at(c));
      if (a.conv) {
        const int entry = a.row_entry[row];
        if (TAPS > 1 && row == a.cu[entry]) {
          // the entry's first row: its window comes from the sequence's state (nothing before position 0)
          const int64_t pos = a.positions[row];
          const float* st = a.state + (int64_t)a.bank_in[entry] * (TAPS - 1) * W;
#pragma unroll
          for (int j = 0; j < TAPS - 1; ++j)
#pragma unroll
            for (int c = 0; c < NC; ++c) {
              const bool live = has[c] && pos - (TAPS - 1) + j >= 0;
              if (live) Chunk<float, VEC>::load(st + (int64_t)j * W + chan[c], &hist[j][c * VEC]);
              else {
#pragma unroll
                for (int e = 0; e < VEC; ++e) hist[j][c * VEC + e] = 0.f;
              }
            }
        }
#pragma unroll
        for (int c = 0; c < C; ++c) {
          auto w = [&](int j) __attribute__((always_inline)) { return kKeepConv ? conv[j][kKeepConv ? c : 0] : conv_at(j, c); };
          float z = w(TAPS - 1) * h[c];
#pragma unroll
          for (int j = 0; j < TAPS - 1; ++j) z = fmaf(w(j), hist[j][c], z);
          o[c] = h[c] + z;
#pragma unroll
          for (int j = 0; j + 1 < TAPS - 1; ++j) hist[j][c] = hist[j + 1][c];
          if (TAPS > 1) hist[kHist - 1][c] = h[c];
        }
        if (TAPS > 1 && mine && row + 1 == a.cu[entry + 1]) {
          float* st = a.state + (int64_t)a.bank_out[entry] * (TAPS - 1) * W;
#pragma unroll
          for (int j = 0; j < TAPS - 1; ++j)
#pragma unroll
            for (int c = 0; c < NC; ++c)
              if (has[c]) Chunk<float, VEC>::store(st + (int64_t)j * W + chan[c], &hist[j][c * VEC]);
        }
      }
      if (mine) {
#pragma unroll
        for (int c = 0; c < NC; ++c) {
          if (!has[c]) continue;
          Chunk<T, VEC>::store(out + (int64_t)row * W + chan[c], &o[c * VEC]);
          if (a.x_out) Chunk<float, VEC>::store(a.x_out + (int64_t)row * W + chan[c], &x[r][c * VEC]);
        }
      }
    }
  }
}

template <typename T, int TAPS>
static int launch_norm_conv(const NormConvArgs& a, dim3 grid, hipStream_t stream) {
  const bool vec = a.width % 4 == 0 && aligned16(a.out) && aligned16(a.x_out) && aligned16(a.x) && aligned16(a.embed) &&
                   aligned16(a.y) && aligned16(a.state);
  const int chunks = vec ? a.width / 4 : a.width;
  const int threads = min(kMaxThreads, (chunks + 63) / 64 * 64);
  const int nc = (chunks + threads - 1) / threads;
  if (nc > 4) return MVLLM_ERR_UNSUPPORTED;
  const dim3 block((unsigned)threads);
  if (vec && nc == 1) norm_conv_kernel<T, TAPS, 4, 1><<<grid, block, 0, stream>>>(a);
  else if (vec) norm_conv_kernel<T, TAPS, 4, 4><<<grid, block, 0, stream>>>(a);
  else norm_conv_kernel<T, TAPS, 1, 4><<<grid, block, 0, stream>>>(a);
  return launch_status();
}

}  // namespace mvllm

using namespace mvllm;

extern "C" int mvllm_norm_conv(void* out, float* x_out, const float* x, const void* embed, const int64_t* tokens,
                               int64_t vocab, const void* y, const float* post, int post_stride, const float* pre,
                               int pre_stride, float eps, const float* conv, int taps, float* state, int64_t num_banks,
                               const int32_t* cu_seqlens, const int32_t* row_entry, const int32_t* bank_in,
                               const int32_t* bank_out, const int64_t* positions, int64_t rows, int width, int dtype,
                               void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || width <= 0 || (post_stride | 1) != 1 || (pre_stride | 1) != 1 || (conv && (taps < 1 || num_banks <= 0)) ||
      (embed && vocab <= 0))
    return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || taps > 8 || rows > (1 << 30)) return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0) return MVLLM_OK;
  if (!out || (!x && !embed) || (embed && !tokens) || !pre || (y && !post)) return MVLLM_ERR_NULL_POINTER;
  if (conv && taps > 1 && (!state || !cu_seqlens || !row_entry || !bank_in || !bank_out || !positions)) return MVLLM_ERR_NULL_POINTER;
  if (conv && (!row_entry || !cu_seqlens)) return MVLLM_ERR_NULL_POINTER;
  if (x_out && (const float*)x_out == x) return MVLLM_ERR_BAD_SHAPE;     // rows in front of a workgroup's own are read again
  NormConvArgs a;
  a.out = out; a.x_out = x_out; a.x = x; a.embed = embed; a.tokens = tokens; a.y = y; a.post = post; a.pre = pre;
  a.conv = conv; a.state = state; a.cu = cu_seqlens; a.row_entry = row_entry; a.bank_in = bank_in; a.bank_out = bank_out;
  a.positions = positions; a.vocab = vocab; a.eps = eps; a.rows = (int)rows; a.width = width;
  a.post_stride = post_stride; a.pre_stride = pre_stride;
  // one row each while that many workgroups fit the chip; long batches in longer walks, so that the rows in front of a
  // walk that are computed twice stay few
  const int halo = conv ? taps - 1 : 0;
  int walk = 1;
  if (rows > 512) {
    walk = (int)((rows + 511) / 512);
    const int cap = 32 - halo;
    walk = walk > cap ? cap : walk;
    walk = (walk + halo + kRowsTogether - 1) / kRowsTogether * kRowsTogether - halo;          // halo + own rows fill whole batches
  }
  a.rows_per_wg = walk;
  const dim3 grid((unsigned)((rows + walk - 1) / walk));
  hipStream_t s = (hipStream_t)stream;
  auto go = [&](auto TAG) -> int {
    using T = decltype(TAG);
    switch (conv ? taps : 1) {
      case 1: return launch_norm_conv<T, 1>(a, grid, s);
      case 2: return launch_norm_conv<T, 2>(a, grid, s);
      case 3: return launch_norm_conv<T, 3>(a, grid, s);
      case 4: return launch_norm_conv<T, 4>(a, grid, s);
      case 5: return launch_norm_conv<T, 5>(a, grid, s);
      case 6: return launch_norm_conv<T, 6>(a, grid, s);
      case 7: return launch_norm_conv<T, 7>(a, grid, s);
      default: return launch_norm_conv<T, 8>(a, grid, s);
    }
  };
  return dtype == MVLLM_F32 ? go(float{}) : go(bf16_t{});
}
