// What stands between two sublayers of a decoder whose residual is several streams (hyper-connections), in one launch:
//     y'   = scale * y                                   (a gain per channel on the sublayer's result)
//     x'_t = sum_s mix[s, t] x_s + out[t] * y'           (all streams at once from the old ones, fp32)
//     h    = rms(sum_t in[t] x'_t) * gain                (what the next sublayer reads; no `in`: the plain sum)
// The sublayer's result is one row y, or what a mixture of experts leaves behind: the sum of `top` rows of `parts` with fp32
// weights (a choice that is no expert counts with the row the mixture read), and a row of a shared expert times the sigmoid of
// one number.  At the front of the model the streams start as
// scaled embedding rows, with a second table indexed by a hash of the token and the one before it:
//     e = embed[token] * embed_scale + bigram[(prev * mul_prev + token * mul_cur) mod buckets]
// (a sequence's first token: row `buckets`).  The token before an entry's first row is part of the sequence's state.
//
// One workgroup per row; a thread keeps the streams' weighted sum of its channels in registers, the streams themselves pass
// through.  They may be updated in place.
#include "row_sums.h"

#pragma clang fp contract(off)

namespace mvllm {

struct StreamNormArgs {
  void* out;                  // [T, out_stride] element type, zeros past the width
  float* x_out;               // [T, S, W] or null
  const float* x;             // [T, S, W]
  const void* y;              // [T, y_stride] element type: the result, or the shared expert's
  const void* parts;          // [*, part_stride] element type
  const int32_t* part_row;    // [T, top] rows of `parts`, or null: row t * top + k
  const float* weights;       // [T, top]
  const int32_t* ids;         // [T, top] or null: a negative one stands for the mixture's input ...
  const void* self;           // ... [T, self_stride] element type
  const float* gate;          // [T, gate_stride]: one logit per row for y, or null
  const float* scale;         // [W] or null
  const float* hc_out;        // [S]
  const float* hc_mix;        // [S, S], from x to
  const float* hc_in;         // [S] or null
  const float* gain;          // [W]
  // the embedding
  const void* embed;          // [vocab, W]
  const void* bigram;         // [buckets + 1, W] or null
  const int64_t* tokens;      // [T]
  int64_t* prev_tokens;       // [banks]
  const int64_t* positions;   // [T]
  const int32_t* cu;          // [entries + 1]
  const int32_t* row_entry;   // [T]
  const int32_t* bank_in;     // [entries]
  const int32_t* bank_out;    // [entries]
  int64_t vocab, buckets, mul_prev, mul_cur;
  int64_t out_stride, y_stride, part_stride, gate_stride, self_stride;
  float embed_scale, eps;
  int width, top;
};

enum { kFromEmbedding = 0, kFromRow = 1, kFromExperts = 2 };

template <typename T, int S, int VEC, int NC, int MODE>
__global__ __launch_bounds__(kMaxThreads) void stream_norm_kernel(const StreamNormArgs a) {
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
  float u[NC][VEC], in[S];
#pragma unroll
  for (int s = 0; s < S; ++s) in[s] = a.hc_in ? a.hc_in[s] : 1.f;
  float* x_out = a.x_out ? a.x_out + row * S * W : nullptr;

  if constexpr (MODE == kFromEmbedding) {
    const int64_t tok = a.tokens[row];
    const T* e_row = reinterpret_cast<const T*>(a.embed) + min(max(tok, (int64_t)0), a.vocab - 1) * W;
    const T* b_row = nullptr;
    const int entry = a.bigram ? a.row_entry[row] : 0;
    if (a.bigram) {
      int64_t at = a.buckets;
      const bool first = row == a.cu[entry];
      if (!first || a.positions[row] > 0) {
        const int64_t prev = first ? a.prev_tokens[a.bank_in[entry]] : a.tokens[row - 1];
        at = (prev * a.mul_prev + tok * a.mul_cur) % a.buckets;
        if (at < 0) at += a.buckets;
      }
      b_row = reinterpret_cast<const T*>(a.bigram) + at * W;
    }
    float total = 0.f;
#pragma unroll
    for (int s = 0; s < S; ++s) total += in[s];
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      float e[VEC], b[VEC];
#pragma unroll
      for (int i = 0; i < VEC; ++i) e[i] = b[i] = 0.f;
      if (has[c]) {
        Chunk<T, VEC>::load(e_row + chan[c], e);
        if (b_row) Chunk<T, VEC>::load(b_row + chan[c], b);
#pragma unroll
        for (int i = 0; i < VEC; ++i) e[i] = e[i] * a.embed_scale + b[i];
        if (x_out) {
#pragma unroll
          for (int s = 0; s < S; ++s) Chunk<float, VEC>::store(x_out + s * W + chan[c], e);
        }
      }
#pragma unroll
      for (int i = 0; i < VEC; ++i) u[c][i] = e[i] * total;
    }
    if (a.bigram) {
      __syncthreads();                              // a decoded row's bank is read and written by this workgroup
      if (tid == 0 && row + 1 == a.cu[entry + 1]) a.prev_tokens[a.bank_out[entry]] = tok;
    }
  } else {
    float mix[S][S], out_w[S];
#pragma unroll
    for (int t = 0; t < S; ++t) {
      out_w[t] = a.hc_out[t];
#pragma unroll
      for (int s = 0; s < S; ++s) mix[s][t] = a.hc_mix[s * S + t];
    }
    const float* x_row = a.x + row * S * W;
    const T* y_row = a.y ? reinterpret_cast<const T*>(a.y) + row * a.y_stride : nullptr;
    float y_gate = 1.f;
    if (MODE == kFromExperts && a.gate && y_row) y_gate = 1.0f / (1.0f + expf(-a.gate[row * a.gate_stride]));
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      float x[S][VEC], y[VEC];
#pragma unroll
      for (int i = 0; i < VEC; ++i) y[i] = u[c][i] = 0.f;
      if (!has[c]) continue;
#pragma unroll
      for (int s = 0; s < S; ++s) Chunk<float, VEC>::load(x_row + s * W + chan[c], x[s]);
      if (y_row) Chunk<T, VEC>::load(y_row + chan[c], y);
      if constexpr (MODE == kFromExperts) {
        float sum[VEC];
#pragma unroll
        for (int i = 0; i < VEC; ++i) sum[i] = 0.f;
        for (int k = 0; k < a.top; ++k) {
          const int64_t at = row * a.top + k;
          const int64_t from = a.part_row ? (int64_t)a.part_row[at] : at;
          const float w = a.weights[at];
          float p[VEC];
          const bool own = a.ids && a.ids[at] < 0;
          const T* p_row = own ? reinterpret_cast<const T*>(a.self) + row * a.self_stride : reinterpret_cast<const T*>(a.parts) + from * a.part_stride;
          Chunk<T, VEC>::load(p_row + chan[c], p);
#pragma unroll
          for (int i = 0; i < VEC; ++i) sum[i] = fmaf(w, p[i], sum[i]);
        }
#pragma unroll
        for (int i = 0; i < VEC; ++i) y[i] = y_row ? fmaf(y_gate, y[i], sum[i]) : sum[i];
      }
      if (a.scale) {
        float g[VEC];
        Chunk<float, VEC>::load(a.scale + chan[c], g);
#pragma unroll
        for (int i = 0; i < VEC; ++i) y[i] *= g[i];
      }
#pragma unroll
      for (int t = 0; t < S; ++t) {
        float z[VEC];
#pragma unroll
        for (int i = 0; i < VEC; ++i) {
          z[i] = out_w[t] * y[i];
#pragma unroll
          for (int s = 0; s < S; ++s) z[i] = fmaf(mix[s][t], x[s][i], z[i]);
          u[c][i] = fmaf(in[t], z[i], u[c][i]);
        }
        if (x_out) Chunk<float, VEC>::store(x_out + t * W + chan[c], z);
      }
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < NC; ++c)
#pragma unroll
    for (int i = 0; i < VEC; ++i) ss = fmaf(u[c][i], u[c][i], ss);
  int flip = 0;
  block_sums<1>(&ss, lds, waves, flip);
  const float inv = 1.0f / sqrtf(ss / (float)W + a.eps);
  T* out = reinterpret_cast<T*>(a.out) + row * a.out_stride;
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    if (!has[c]) continue;
    float g[VEC], o[VEC];
    Chunk<float, VEC>::load(a.gain + chan[c], g);
#pragma unroll
    for (int i = 0; i < VEC; ++i) o[i] = u[c][i] * inv * g[i];
    Chunk<T, VEC>::store(out + chan[c], o);
  }
  for (int64_t c = W + tid; c < a.out_stride; c += blockDim.x) out[c] = from_float<T>(0.f);
}

template <typename T, int S, int MODE>
static int launch_stream_norm(const StreamNormArgs& a, int rows, hipStream_t stream) {
  const int n = sizeof(T) == 4 ? 4 : 8;            // rows of the element type start on 8 or 16 bytes
  const bool vec = a.width % 4 == 0 && (a.out_stride * (int64_t)sizeof(T)) % n == 0 && (a.y_stride * (int64_t)sizeof(T)) % n == 0 &&
                   (a.part_stride * (int64_t)sizeof(T)) % n == 0 && (a.self_stride * (int64_t)sizeof(T)) % n == 0 && aligned16(a.self) && aligned16(a.out) && aligned16(a.x_out) && aligned16(a.x) &&
                   aligned16(a.y) && aligned16(a.parts) && aligned16(a.scale) && aligned16(a.gain) && aligned16(a.embed) && aligned16(a.bigram);
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
  if (vec && nc == 1) stream_norm_kernel<T, S, 4, 1, MODE><<<grid, block, 0, stream>>>(a);
  else if (vec && nc == 2) stream_norm_kernel<T, S, 4, 2, MODE><<<grid, block, 0, stream>>>(a);
  else if (vec) stream_norm_kernel<T, S, 4, 4, MODE><<<grid, block, 0, stream>>>(a);
  else stream_norm_kernel<T, S, 1, 4, MODE><<<grid, block, 0, stream>>>(a);
  return launch_status();
}

template <typename T, int MODE>
static int launch_streams(const StreamNormArgs& a, int rows, int streams, hipStream_t stream) {
  switch (streams) {
    case 1: return launch_stream_norm<T, 1, MODE>(a, rows, stream);
    case 2: return launch_stream_norm<T, 2, MODE>(a, rows, stream);
    case 3: return launch_stream_norm<T, 3, MODE>(a, rows, stream);
    case 4: return launch_stream_norm<T, 4, MODE>(a, rows, stream);
    case 5: return launch_stream_norm<T, 5, MODE>(a, rows, stream);
    case 6: return launch_stream_norm<T, 6, MODE>(a, rows, stream);
    case 7: return launch_stream_norm<T, 7, MODE>(a, rows, stream);
    case 8: return launch_stream_norm<T, 8, MODE>(a, rows, stream);
    default: return MVLLM_ERR_UNSUPPORTED;
  }
}

static int check_common(void* out, int64_t out_stride, const float* gain, int64_t rows, int streams, int width, int dtype) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || width <= 0 || streams <= 0 || out_stride < width) return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || streams > 8 || rows > (1 << 30)) return MVLLM_ERR_UNSUPPORTED;
  if (rows > 0 && (!out || !gain)) return MVLLM_ERR_NULL_POINTER;
  return MVLLM_OK;
}

}  // namespace mvllm

using namespace mvllm;

extern "C" int mvllm_stream_embed_norm(void* out, int64_t out_row_stride, float* x_out, const void* embed, int64_t vocab,
                                       float embed_scale, const void* bigram, int64_t buckets, int64_t mul_prev,
                                       int64_t mul_cur, int64_t* prev_tokens, const int64_t* tokens,
                                       const int64_t* positions, const int32_t* cu_seqlens, const int32_t* row_entry,
                                       const int32_t* bank_in, const int32_t* bank_out, const float* hc_in,
                                       const float* gain, float eps, int64_t rows, int streams, int width, int dtype,
                                       void* stream) {
  const int st = check_common(out, out_row_stride, gain, rows, streams, width, dtype);
  if (st != MVLLM_OK) return st;
  if (vocab <= 0 || (bigram && buckets <= 0)) return MVLLM_ERR_BAD_SHAPE;
  if (rows == 0) return MVLLM_OK;
  if (!embed || !tokens) return MVLLM_ERR_NULL_POINTER;
  if (bigram && (!prev_tokens || !positions || !cu_seqlens || !row_entry || !bank_in || !bank_out)) return MVLLM_ERR_NULL_POINTER;
  StreamNormArgs a = {};
  a.out = out; a.out_stride = out_row_stride; a.x_out = x_out; a.embed = embed; a.vocab = vocab; a.embed_scale = embed_scale;
  a.bigram = bigram; a.buckets = buckets; a.mul_prev = mul_prev; a.mul_cur = mul_cur; a.prev_tokens = prev_tokens;
  a.tokens = tokens; a.positions = positions; a.cu = cu_seqlens; a.row_entry = row_entry; a.bank_in = bank_in;
  a.bank_out = bank_out; a.hc_in = hc_in; a.gain = gain; a.eps = eps; a.width = width;
  hipStream_t s = (hipStream_t)stream;
  return dtype == MVLLM_F32 ? launch_streams<float, kFromEmbedding>(a, (int)rows, streams, s)
                            : launch_streams<bf16_t, kFromEmbedding>(a, (int)rows, streams, s);
}

extern "C" int mvllm_stream_norm_identity(void* out, int64_t out_row_stride, float* x_out, const float* x, const void* y,
                                          int64_t y_row_stride, const void* parts, int64_t part_row_stride,
                                          const int32_t* part_row, const float* weights, int top, const int32_t* ids,
                                          const void* self, int64_t self_row_stride, const float* gate,
                                          int64_t gate_row_stride, const float* scale, const float* hc_out,
                                          const float* hc_mix, const float* hc_in, const float* gain, float eps,
                                          int64_t rows, int streams, int width, int dtype, void* stream) {
  const int st = check_common(out, out_row_stride, gain, rows, streams, width, dtype);
  if (st != MVLLM_OK) return st;
  if ((y && y_row_stride < width) || (parts && (part_row_stride < width || top <= 0)) || (gate && gate_row_stride <= 0) || (ids && self_row_stride < width)) return MVLLM_ERR_BAD_SHAPE;
  if (rows == 0) return MVLLM_OK;
  if (!x || !hc_out || !hc_mix || (!y && !parts) || (parts && !weights) || (ids && !self)) return MVLLM_ERR_NULL_POINTER;
  StreamNormArgs a = {};
  a.out = out; a.out_stride = out_row_stride; a.x_out = x_out; a.x = x; a.y = y; a.y_stride = y_row_stride; a.parts = parts;
  a.part_stride = part_row_stride; a.part_row = part_row; a.weights = weights; a.top = top; a.gate = gate;
  a.gate_stride = gate_row_stride; a.scale = scale; a.hc_out = hc_out; a.hc_mix = hc_mix; a.hc_in = hc_in; a.gain = gain;
  a.eps = eps; a.width = width; a.ids = ids; a.self = self; a.self_stride = self_row_stride;
  hipStream_t s = (hipStream_t)stream;
  if (parts)
    return dtype == MVLLM_F32 ? launch_streams<float, kFromExperts>(a, (int)rows, streams, s)
                              : launch_streams<bf16_t, kFromExperts>(a, (int)rows, streams, s);
  return dtype == MVLLM_F32 ? launch_streams<float, kFromRow>(a, (int)rows, streams, s)
                            : launch_streams<bf16_t, kFromRow>(a, (int)rows, streams, s);
}

extern "C" int mvllm_stream_norm(void* out, int64_t out_row_stride, float* x_out, const float* x, const void* y,
                                 int64_t y_row_stride, const void* parts, int64_t part_row_stride,
                                 const int32_t* part_row, const float* weights, int top, const float* gate,
                                 int64_t gate_row_stride, const float* scale, const float* hc_out, const float* hc_mix,
                                 const float* hc_in, const float* gain, float eps, int64_t rows, int streams, int width,
                                 int dtype, void* stream) {
  return mvllm_stream_norm_identity(out, out_row_stride, x_out, x, y, y_row_stride, parts, part_row_stride, part_row, weights, top,
                                    nullptr, nullptr, 0, gate, gate_row_stride, scale, hc_out, hc_mix, hc_in, gain, eps, rows, streams,
                                    width, dtype, stream);
}
