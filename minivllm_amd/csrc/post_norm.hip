// What stands behind a sublayer of a decoder that norms what its sublayers return and nothing else, in one launch:
//     x' = x + norm(y) * gain                    (fp32)
//     h  = x', or norm(x') * final_gain          (what the next sublayer, or the head, reads)
// norm takes the mean off first (layer norm) or does not (root mean square).  As the model's first launch it makes
//     x' = embed[token] * scale.
// One workgroup per row, its channels in registers; sums of deviations, not of squares, so that a mean far from zero costs
// no digits.  x may be updated in place.
#include "row_sums.h"

#pragma clang fp contract(off)

namespace mvllm {

struct PostNormArgs {
  void* out;                  // [T, out_stride] element type, zeros past the width
  float* x_out;               // [T, W] or null
  const float* x;             // [T, W]
  const void* y;              // [T, y_stride] element type
  const float* gain;          // [W]
  const float* final_gain;    // [W] or null
  const void* embed;          // [vocab, W] element type
  const int64_t* tokens;      // [T] or null: the embedding instead of x and y
  int64_t vocab, out_stride, y_stride;
  float embed_scale, eps;
  int width, centred;
};

template <typename T, int VEC, int NC, bool EMBED>
__global__ __launch_bounds__(kMaxThreads) void post_norm_kernel(const PostNormArgs a) {
  __shared__ __attribute__((aligned(16))) float lds[2 * (kMaxThreads / 16)];
  const int64_t row = blockIdx.x;
  const int W = a.width, tid = threadIdx.x, waves = blockDim.x >> 6;
  int chan[NC];
  bool has[NC];
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    chan[c] = (tid + c * blockDim.x) * VEC;
    has[c] = chan[c] < W;
  }
  int flip = 0;
  // 1 / sqrt(mean of squares + eps), and the mean taken off before that
  auto normed = [&](float (&v)[NC][VEC]) __attribute__((always_inline)) {
    if (a.centred) {
      float sum = 0.f;
#pragma unroll
      for (int c = 0; c < NC; ++c)
#pragma unroll
        for (int i = 0; i < VEC; ++i) sum += v[c][i];                  // channels that are not there are zeros
      block_sums<1>(&sum, lds, waves, flip);
      const float mean = sum / (float)W;
#pragma unroll
      for (int c = 0; c < NC; ++c)
#pragma unroll
        for (int i = 0; i < VEC; ++i) v[c][i] = has[c] ? v[c][i] - mean : 0.f;
    }
    float ss = 0.f;
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int i = 0; i < VEC; ++i) ss = fmaf(v[c][i], v[c][i], ss);
    block_sums<1>(&ss, lds, waves, flip);
    return 1.0f / sqrtf(ss / (float)W + a.eps);
  };

  float u[NC][VEC];
  if constexpr (EMBED) {
    const T* e_row = reinterpret_cast<const T*>(a.embed) + min(max(a.tokens[row], (int64_t)0), a.vocab - 1) * W;
#pragma unroll
    for (int c = 0; c < NC; ++c) {
#pragma unroll
      for (int i = 0; i < VEC; ++i) u[c][i] = 0.f;
      if (!has[c]) continue;
      Chunk<T, VEC>::load(e_row + chan[c], u[c]);
#pragma unroll
      for (int i = 0; i < VEC; ++i) u[c][i] *= a.embed_scale;
    }
  } else {
    const float* x_row = a.x + row * W;
    const T* y_row = reinterpret_cast<const T*>(a.y) + row * a.y_stride;
    float x[NC][VEC], g[NC][VEC];
#pragma unroll
    for (int c = 0; c < NC; ++c) {
#pragma unroll
      for (int i = 0; i < VEC; ++i) u[c][i] = x[c][i] = g[c][i] = 0.f;
      if (!has[c]) continue;
      Chunk<T, VEC>::load(y_row + chan[c], u[c]);
      Chunk<float, VEC>::load(x_row + chan[c], x[c]);
      Chunk<float, VEC>::load(a.gain + chan[c], g[c]);
    }
    const float inv = normed(u);
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int i = 0; i < VEC; ++i) u[c][i] = fmaf(u[c][i] * inv, g[c][i], x[c][i]);
  }
  if (a.x_out) {
#pragma unroll
    for (int c = 0; c < NC; ++c)
      if (has[c]) Chunk<float, VEC>::store(a.x_out + row * W + chan[c], u[c]);
  }
  if (a.final_gain) {
    const float inv = normed(u);
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      if (!has[c]) continue;
      float g[VEC];
      Chunk<float, VEC>::load(a.final_gain + chan[c], g);
#pragma unroll
      for (int i = 0; i < VEC; ++i) u[c][i] = u[c][i] * inv * g[i];
    }
  }
  T* out = reinterpret_cast<T*>(a.out) + row * a.out_stride;
#pragma unroll
  for (int c = 0; c < NC; ++c)
    if (has[c]) Chunk<T, VEC>::store(out + chan[c], u[c]);
  for (int64_t c = W + tid; c < a.out_stride; c += blockDim.x) out[c] = from_float<T>(0.f);
}

template <typename T, bool EMBED>
static int launch_post_norm(const PostNormArgs& a, int rows, hipStream_t stream) {
  const int n = sizeof(T) == 4 ? 4 : 8;            // rows of the element type start on 8 or 16 bytes
  const bool vec = a.width % 4 == 0 && (a.out_stride * (int64_t)sizeof(T)) % n == 0 && (a.y_stride * (int64_t)sizeof(T)) % n == 0 &&
                   aligned16(a.out) && aligned16(a.x_out) && aligned16(a.x) && aligned16(a.y) && aligned16(a.gain) &&
                   aligned16(a.final_gain) && aligned16(a.embed);
  const int chunks = vec ? a.width / 4 : a.width;
  // few rows: short threads; many: 256 threads with several chunks each, so that a row's loads overlap
  const int most = rows <= 512 ? kMaxThreads : 256;
  int threads = min(most, (chunks + 63) / 64 * 64);
  int nc = (chunks + threads - 1) / threads;
  if (nc > 4) {
    threads = kMaxThreads;
    nc = (chunks + threads - 1) / threads;
  }
  if (nc > 4) return MVLLM_ERR_UNSUPPORTED;
  const dim3 grid((unsigned)rows), block((unsigned)threads);
  if (vec && nc == 1) post_norm_kernel<T, 4, 1, EMBED><<<grid, block, 0, stream>>>(a);
  else if (vec && nc == 2) post_norm_kernel<T, 4, 2, EMBED><<<grid, block, 0, stream>>>(a);
  else if (vec) post_norm_kernel<T, 4, 4, EMBED><<<grid, block, 0, stream>>>(a);
  else post_norm_kernel<T, 1, 4, EMBED><<<grid, block, 0, stream>>>(a);
  return launch_status();
}

}  // namespace mvllm

using namespace mvllm;

extern "C" int mvllm_post_norm(void* out, int64_t out_row_stride, float* x_out, const float* x, const void* y,
                               int64_t y_row_stride, const float* gain, const float* final_gain, float eps, int centred,
                               int64_t rows, int width, int dtype, void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || width <= 0 || out_row_stride < width || y_row_stride < width) return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || rows > (1 << 30)) return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0) return MVLLM_OK;
  if (!out || !x || !y || !gain) return MVLLM_ERR_NULL_POINTER;
  PostNormArgs a = {};
  a.out = out; a.out_stride = out_row_stride; a.x_out = x_out; a.x = x; a.y = y; a.y_stride = y_row_stride; a.gain = gain;
  a.final_gain = final_gain; a.eps = eps; a.centred = centred; a.width = width;
  return dtype == MVLLM_F32 ? launch_post_norm<float, false>(a, (int)rows, (hipStream_t)stream)
                            : launch_post_norm<bf16_t, false>(a, (int)rows, (hipStream_t)stream);
}

extern "C" int mvllm_embed_rows(void* out, int64_t out_row_stride, float* x_out, const void* embed, int64_t vocab, float scale,
                                const int64_t* tokens, int64_t rows, int width, int dtype, void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || width <= 0 || vocab <= 0 || out_row_stride < width) return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || rows > (1 << 30)) return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0) return MVLLM_OK;
  if (!out || !embed || !tokens) return MVLLM_ERR_NULL_POINTER;
  PostNormArgs a = {};
  a.out = out; a.out_stride = out_row_stride; a.x_out = x_out; a.embed = embed; a.vocab = vocab; a.embed_scale = scale;
  a.tokens = tokens; a.width = width;
  return dtype == MVLLM_F32 ? launch_post_norm<float, true>(a, (int)rows, (hipStream_t)stream)
                            : launch_post_norm<bf16_t, true>(a, (int)rows, (hipStream_t)stream);
}
