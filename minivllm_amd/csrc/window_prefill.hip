// Windowed prefill: entry point, tiled kernels for values that are the keys, and the kernel for every other size and for fp32.
#include "window_prefill.h"

namespace mvllm {

// Any size up to 64 NE per part: a query row and head per wave, one key at a time (four in flight), lanes split the columns.
template <typename T, int NE>
__global__ __launch_bounds__(256) void window_prefill_any_kernel(const WindowPrefillArgs a) {
  int seq_start, seq_len, row0, seq;
  if (!locate_tile(a.cu_q, a.num_seqs, blockIdx.x, 4, seq_start, seq_len, row0, seq)) return;
  const int lane = threadIdx.x & 63, r = row0 + (threadIdx.x >> 6), h = blockIdx.y, g = h / (a.heads / a.kv_heads);
  if (r >= seq_len) return;
  const int k_start = a.cu_k[seq], kv_len = a.cu_k[seq + 1] - k_start, pos = kv_len - seq_len + r;
  const int first = a.window > 0 ? max(pos - a.window + 1, 0) : 0;
  const int64_t t = (int64_t)seq_start + r;
  const T* q = reinterpret_cast<const T*>(a.q) + t * a.q_row + (int64_t)h * a.q_head;
  const T* k = reinterpret_cast<const T*>(a.k) + (int64_t)k_start * a.k_row + (int64_t)g * a.k_head;
  const T* k2 = a.k2 ? reinterpret_cast<const T*>(a.k2) + (int64_t)k_start * a.k2_row : nullptr;
  const T* v = a.v ? reinterpret_cast<const T*>(a.v) + (int64_t)k_start * a.v_row + (int64_t)g * a.v_head : nullptr;
  const float scale = a.scale_log2 * prefill_temperature(a, t), slope = a.slopes ? a.slopes[h] * kLog2e : 0.f;
  float qv[NE], qr[NE], o[NE];
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int c = lane + 64 * i;
    qv[i] = c < a.dim ? to_float(q[c]) * scale : 0.f;
    qr[i] = k2 && c < a.rot ? to_float(q[a.dim + c]) * scale : 0.f;
    o[i] = 0.f;
  }
  float m = -INFINITY, l = 0.f;
  for (int j0 = first; j0 <= pos; j0 += 4) {
    float s[4], x[4][NE], most = m;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int64_t j = min(j0 + e, pos);
      s[e] = 0.f;
#pragma unroll
      for (int i = 0; i < NE; ++i) {
        const int c = lane + 64 * i;
        const float kv = c < a.dim ? to_float(k[j * a.k_row + c]) : 0.f;
        s[e] = fmaf(qv[i], kv, s[e]);
        if (k2 && c < a.rot) s[e] = fmaf(qr[i], to_float(k2[j * a.k2_row + c]), s[e]);
        x[e][i] = !v ? kv : c < a.dim ? to_float(v[j * a.v_row + c]) : 0.f;
      }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      s[e] = j0 + e <= pos ? wave_sum(s[e]) - slope * (float)(pos - j0 - e) : -INFINITY;
      most = fmaxf(most, s[e]);
    }
    const float keep = exp2f(m - most);              // the first key is always seen: `most` is finite
    m = most;
    l *= keep;
#pragma unroll
    for (int i = 0; i < NE; ++i) o[i] *= keep;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float p = exp2f(s[e] - m);
      l += p;
#pragma unroll
      for (int i = 0; i < NE; ++i) o[i] = fmaf(p, x[e][i], o[i]);
    }
  }
  const float inv = 1.f / l;
  T* out = reinterpret_cast<T*>(a.out) + t * a.out_row + (int64_t)h * a.out_head;
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int c = lane + 64 * i;
    if (c >= a.dim) continue;
    float x = o[i] * inv;
    if (a.gate) x /= 1.f + expf(-to_float(reinterpret_cast<const T*>(a.gate)[t * a.gate_row + (int64_t)h * a.gate_head + (a.gate_head == 1 ? 0 : c)]));
    out[c] = from_float<T>(x);
  }
}

template <typename T>
static int launch_any(const WindowPrefillArgs& a, hipStream_t s) {
  const int widest = a.dim > a.rot ? a.dim : a.rot;
  const dim3 grid((unsigned)(a.total_q / 4 + a.num_seqs), (unsigned)a.heads), block(256);
  if (widest <= 64) window_prefill_any_kernel<T, 1><<<grid, block, 0, s>>>(a);
  else if (widest <= 128) window_prefill_any_kernel<T, 2><<<grid, block, 0, s>>>(a);
  else if (widest <= 256) window_prefill_any_kernel<T, 4><<<grid, block, 0, s>>>(a);
  else if (widest <= 512) window_prefill_any_kernel<T, 8><<<grid, block, 0, s>>>(a);
  else return MVLLM_ERR_UNSUPPORTED;
  return launch_status();
}

static int launch_shared(const WindowPrefillArgs& a, hipStream_t s) {
  switch (a.dim) {
    case 32: return launch_window_prefill<2, 0, 1, true>(a, s);
    case 64: return launch_window_prefill<4, 0, 2, true>(a, s);
    case 96: return launch_window_prefill<6, 0, 3, true>(a, s);
    case 128: return launch_window_prefill<8, 0, 4, true>(a, s);
    case 192: return launch_window_prefill<12, 0, 6, true>(a, s);
    case 256: return launch_window_prefill<16, 0, 8, true>(a, s);
    default: return kNoTiles;
  }
}

__attribute__((weak)) int launch_window_prefill_parts(const WindowPrefillArgs&, hipStream_t) { return kNoTiles; }
__attribute__((weak)) int launch_window_prefill_heads(const WindowPrefillArgs&, hipStream_t) { return kNoTiles; }

}  // namespace mvllm

using namespace mvllm;

extern "C" int mvllm_window_prefill(void* out, int64_t out_row_stride, int64_t out_head_stride, const void* q,
                                    int64_t q_row_stride, int64_t q_head_stride, const void* k, int64_t k_row_stride,
                                    int64_t k_head_stride, const void* k2, int64_t k2_row_stride, const void* v,
                                    int64_t v_row_stride, int64_t v_head_stride, const void* gate,
                                    int64_t gate_row_stride, int64_t gate_head_stride, const int32_t* cu_q,
                                    const int32_t* cu_k, const int64_t* positions, const float* slopes, int num_seqs,
                                    int64_t total_q, int num_heads, int num_kv_heads, int dim, int rot, int window,
                                    float scale, float temp_coef, float temp_every, int dtype, void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (num_seqs < 0 || total_q < 0 || num_heads <= 0 || num_kv_heads <= 0 || num_heads % num_kv_heads != 0 || dim <= 0 || rot < 0 ||
      window < 0 || (k2 == nullptr) != (rot == 0) || q_head_stride < dim + rot || out_head_stride < dim || k_row_stride < dim ||
      (v && v_row_stride < dim) || (k2 && k2_row_stride < rot) || (gate && gate_head_stride != 1 && gate_head_stride < dim) || !(temp_every >= 0.f))
    return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || num_heads > 65535 || total_q > ((int64_t)1 << 30)) return MVLLM_ERR_UNSUPPORTED;
  if (num_seqs == 0 || total_q == 0) return MVLLM_OK;
  if (!out || !q || !k || !cu_q || !cu_k || (temp_every > 0.f && !positions)) return MVLLM_ERR_NULL_POINTER;
  WindowPrefillArgs a = {};
  a.out = out; a.q = q; a.k = k; a.k2 = k2; a.v = v; a.gate = gate; a.cu_q = cu_q; a.cu_k = cu_k; a.positions = positions;
  a.slopes = slopes; a.out_row = out_row_stride; a.out_head = out_head_stride; a.q_row = q_row_stride; a.q_head = q_head_stride;
  a.k_row = k_row_stride; a.k_head = k_head_stride; a.k2_row = k2_row_stride; a.v_row = v_row_stride; a.v_head = v_head_stride;
  a.gate_row = gate_row_stride; a.gate_head = gate_head_stride; a.total_q = total_q; a.num_seqs = num_seqs; a.heads = num_heads;
  a.kv_heads = num_kv_heads; a.dim = dim; a.rot = rot; a.window = window; a.scale_log2 = scale * kLog2e;
  a.temp_coef = temp_coef; a.temp_every = temp_every;
  hipStream_t s = (hipStream_t)stream;
  const bool one_gate = gate_head_stride == 1;       // read number by number
  const int64_t strides[] = {out_row_stride, out_head_stride, q_row_stride, q_head_stride, k_row_stride, k_head_stride, k2_row_stride,
                             v_row_stride, v_head_stride, one_gate ? 0 : gate_row_stride, one_gate ? 0 : gate_head_stride};
  bool tiles = dtype == MVLLM_BF16 && aligned16(out) && aligned16(q) && aligned16(k) && aligned16(k2) && aligned16(v) && (one_gate || aligned16(gate)) &&
               k_row_stride < (1 << 24) && k2_row_stride < (1 << 24) && v_row_stride < (1 << 24) && (v || !k2) && !(v && slopes);
  for (int64_t x : strides) tiles = tiles && x % 8 == 0;
  const int st = !tiles ? kNoTiles : k2 ? launch_window_prefill_parts(a, s) : v ? launch_window_prefill_heads(a, s) : launch_shared(a, s);
  if (st != kNoTiles) return st;
  return dtype == MVLLM_F32 ? launch_any<float>(a, s) : launch_any<bf16_t>(a, s);
}
