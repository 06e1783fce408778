// Single query rows over a paged ring of the last tokens whose cached rows are keys and values at once (latents with a rotated
// part, or keys that are their own values) or a key and its value (kernels in latent_decode.h).  What the windowed prefill (window_prefill.hip) does
// for long portions this does for decoded tokens and short ones:
//     score = scale * temperature(p) * q . k - slope_h * distance      for distance < window
// and the result times sigmoid(gate), where there is one.
#include "latent_decode.h"

namespace mvllm {
__attribute__((weak)) int launch_decode_split(const LatentDecodeArgs&, int, hipStream_t) { return kNotBuilt; }
}  // namespace mvllm

using namespace mvllm;

extern "C" size_t mvllm_window_decode_workspace_bytes(int rows, int num_heads, int num_kv_heads, int padded, int values,
                                                      int64_t max_keys, int dtype) {
  if (rows <= 0 || num_heads <= 0 || num_kv_heads <= 0 || padded <= 0 || values <= 0 || max_keys <= 0) return 0;
  const int parts = plan_parts(rows, num_heads, num_kv_heads, padded, max_keys, dtype);
  return parts == 1 ? 0 : (size_t)rows * parts * num_heads * ((size_t)values + 2) * sizeof(float);
}

// Rows of `padded` key columns; the values are their first `values` columns (value_col 0) or stand behind them.
static int window_decode(void* out, int64_t out_row_stride, int64_t out_head_stride, const void* q, int64_t q_row_stride,
                         int64_t q_head_stride, const void* cache, const int32_t* block_tables, int table_width,
                         const int32_t* row_entry, const int64_t* lens, const float* slopes, const void* gate,
                         int64_t gate_row_stride, int64_t gate_head_stride, int rows, int num_heads, int num_kv_heads, int padded,
                         int values, int value_col, int block_size, int64_t num_blocks, int window, int ring, float scale,
                         float temp_coef, float temp_every, int dtype, void* workspace, size_t workspace_bytes, void* stream) {
  if (dtype_size(dtype) == 0) return MVLLM_ERR_BAD_DTYPE;
  if (rows < 0 || num_heads <= 0 || num_kv_heads <= 0 || num_heads % num_kv_heads != 0 || padded <= 0 || padded % 32 != 0 ||
      values <= 0 || values % 32 != 0 || table_width <= 0 || block_size <= 0 || num_blocks <= 0 ||
      (int64_t)table_width * block_size >= (int64_t)1 << 31 || window < 0 || ring < 0 || (ring > 0 && window > ring) ||
      q_head_stride < padded || out_head_stride < values || (gate && gate_head_stride != 1 && gate_head_stride < values) || !(temp_every >= 0.f))
    return MVLLM_ERR_BAD_SHAPE;
  if (dtype == MVLLM_F16 || padded > 2048 || values > 2048 || num_heads > 65535 || rows > 65535 || q_row_stride % 8 != 0 ||
      q_head_stride % 8 != 0 || out_row_stride % 4 != 0 || out_head_stride % 4 != 0 ||
      (gate_head_stride != 1 && (gate_row_stride % 4 != 0 || gate_head_stride % 4 != 0)))
    return MVLLM_ERR_UNSUPPORTED;
  if (rows == 0) return MVLLM_OK;
  if (!out || !q || !cache || !block_tables || !row_entry || !lens) return MVLLM_ERR_NULL_POINTER;
  if (!aligned16(out) || !aligned16(q) || !aligned16(cache) || (gate_head_stride != 1 && !aligned16(gate))) return MVLLM_ERR_MISALIGNED;
  LatentDecodeArgs a = {};
  a.out = out; a.q = q; a.cache = cache; a.tables = block_tables; a.row_entry = row_entry; a.lens = lens;
  a.num_blocks = num_blocks; a.table_width = table_width; a.block_size = block_size; a.heads = num_heads;
  a.kv_heads = num_kv_heads; a.padded = padded; a.values = values; a.value_col = value_col;
  a.row = value_col > 0 ? padded + values : padded; a.q_row = q_row_stride; a.q_head = q_head_stride;
  a.out_row = out_row_stride; a.out_head = out_head_stride; a.scale_log2 = scale * kLog2e; a.slopes = slopes; a.gate = gate;
  a.gate_row = gate_row_stride; a.gate_head = gate_head_stride; a.window = window; a.ring = ring;
  a.temp_coef = temp_coef; a.temp_every = temp_every;
  const int64_t max_keys = (int64_t)table_width * block_size;
  a.parts = plan_parts(rows, num_heads, num_kv_heads, a.row, max_keys, dtype);
  if (a.parts > 1) {
    if (!workspace || !aligned16(workspace) || workspace_bytes < mvllm_window_decode_workspace_bytes(rows, num_heads, num_kv_heads, a.row, values, max_keys, dtype))
      return MVLLM_ERR_WORKSPACE;
    a.part_o = reinterpret_cast<float*>(workspace);
    a.part_ml = reinterpret_cast<float2*>(a.part_o + (int64_t)rows * a.parts * num_heads * values);
  }
  return launch_decode<true>(a, rows, dtype, (hipStream_t)stream);
}

extern "C" int mvllm_window_decode(void* out, int64_t out_row_stride, int64_t out_head_stride, const void* q,
                                   int64_t q_row_stride, int64_t q_head_stride, const void* cache,
                                   const int32_t* block_tables, int table_width, const int32_t* row_entry,
                                   const int64_t* lens, const float* slopes, const void* gate, int64_t gate_row_stride,
                                   int64_t gate_head_stride, int rows, int num_heads, int num_kv_heads, int padded,
                                   int values, int block_size, int64_t num_blocks, int window, int ring, float scale,
                                   float temp_coef, float temp_every, int dtype, void* workspace, size_t workspace_bytes,
                                   void* stream) {
  if (values != padded && !(padded == 576 && values == 512)) return MVLLM_ERR_BAD_SHAPE;
  return window_decode(out, out_row_stride, out_head_stride, q, q_row_stride, q_head_stride, cache, block_tables, table_width,
                       row_entry, lens, slopes, gate, gate_row_stride, gate_head_stride, rows, num_heads, num_kv_heads, padded,
                       values, 0, block_size, num_blocks, window, ring, scale, temp_coef, temp_every, dtype, workspace,
                       workspace_bytes, stream);
}

extern "C" int mvllm_window_decode_split(void* out, int64_t out_row_stride, int64_t out_head_stride, const void* q,
                                         int64_t q_row_stride, int64_t q_head_stride, const void* cache,
                                         const int32_t* block_tables, int table_width, const int32_t* row_entry,
                                         const int64_t* lens, const float* slopes, const void* gate, int64_t gate_row_stride,
                                         int64_t gate_head_stride, int rows, int num_heads, int num_kv_heads, int keys,
                                         int values, int block_size, int64_t num_blocks, int window, int ring, float scale,
                                         float temp_coef, float temp_every, int dtype, void* workspace, size_t workspace_bytes,
                                         void* stream) {
  return window_decode(out, out_row_stride, out_head_stride, q, q_row_stride, q_head_stride, cache, block_tables, table_width,
                       row_entry, lens, slopes, gate, gate_row_stride, gate_head_stride, rows, num_heads, num_kv_heads, keys,
                       values, keys, block_size, num_blocks, window, ring, scale, temp_coef, temp_every, dtype, workspace,
                       workspace_bytes, stream);
}
