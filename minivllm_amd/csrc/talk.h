// Attention whose heads' scores are mixed before the softmax:
//     s_h(i, j) = sum_g talk[h, g] q_g(i) . k_kv(g)(j),   p_h = softmax_j(s_h) with an optional sink,   o_h = p_h v_kv(h)
// so that no head's weights are known before every head's scores are.  Queries carry the score scale and log2 e: scores are
// exponents of two as they come.  A row's keys are the tokens of its piece up to its own, cached (block tables, the earlier
// tokens of the piece in front) or packed beside the queries.
#pragma once
#include "latent_decode.h"

#pragma clang fp contract(off)

namespace mvllm {

struct TalkArgs {
  void* out;                  // row out_rows[t] (null: t) at out_row, head h at h * out_head
  const void* q;              // [rows, heads, dim]
  const void* k;              // packed [*, kv_heads, dim], or a cache [num_blocks, block_size, kv_heads, dim]
  const void* v;
  const int32_t* out_rows;
  const int32_t* cu_q;        // [num_seqs + 1]; null: single rows, `lens` keys each
  const int32_t* cu_k;        // [num_seqs + 1]; null: the queries' (packed)
  const int32_t* tables;      // [num_seqs or rows, table_width]; null: packed
  const int64_t* lens;        // [rows]
  const float* talk;          // [heads, heads]
  const float* sinks;         // [heads] or null, natural units
  float* part_o;              // [rows, parts, heads, dim] (single rows, parts > 1)
  float2* part_ml;            // [rows, parts, heads]: maximum (base 2), sum
  int64_t out_row, out_head, total_q, num_blocks;
  int num_seqs, heads, kv_heads, dim, table_width, block_size, parts;
  // the tiled prefill, filled in by its launcher: item order; query heads per kv head, pieces of them and 65536 / pieces_per_kv + 1
  int tiles_x, heads_y, band_bits, band_shift, per, pieces, pieces_per_kv;
  unsigned piece_magic;
};

// Heads, `most` at a time, that share a kv head: what one wave makes raw scores of.
struct TalkPieces {
  int per_kv, count;
  __host__ __device__ TalkPieces(int heads, int kv_heads, int most)
      : per_kv((heads / kv_heads + most - 1) / most), count(kv_heads * ((heads / kv_heads + most - 1) / most)) {}
};

int launch_talk_prefill(const TalkArgs& a, hipStream_t stream);      // talk_prefill.hip; kNotBuilt where it takes nothing
int launch_talk_decode(const TalkArgs& a, int rows, hipStream_t stream);      // talk_decode.hip

}  // namespace mvllm
