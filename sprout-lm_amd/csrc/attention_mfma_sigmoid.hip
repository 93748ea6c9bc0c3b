// bfloat16 attention whose weights are sigmoid(score + bias), not normalised: the instantiations.
#include "attention_mfma.h"

namespace sprout {

int attention_mfma_wide_sigmoid(hipStream_t s, const void* q, int q_stride, const void* k_pool, const void* v_pool,
                                const int32_t* block_tables, int max_blocks, const int32_t* q_start, const int32_t* q_len,
                                const int32_t* ctx_len, const int32_t* tiles, int n_tiles, const int32_t* decode_seqs,
                                int n_decode, int max_decode_ctx, int max_tile_ctx, int mean_tile_walk, float* workspace,
                                void* out, int nq, int nkv, int hd, int page_size, int num_pages, ScoreStage st, float scale);

int attention_mfma_sigmoid(hipStream_t s, const void* q, int q_stride, const void* k_pool, const void* v_pool,
                   const int32_t* block_tables, int max_blocks, const int32_t* q_start, const int32_t* q_len,
                   const int32_t* ctx_len, const int32_t* tiles, int n_tiles, const int32_t* decode_seqs, int n_decode,
                   int max_decode_ctx, int max_tile_ctx, int mean_tile_walk, float* workspace, void* out, int nq, int nkv,
                   int hd, int page_size, int num_pages, ScoreStage st, float scale) {
#define SP_MFMA(DT)                                                                                              \
  case DT:                                                                                                       \
    return launch_mfma<DT, true>(s, q, q_stride, k_pool, v_pool, block_tables, max_blocks, q_start, q_len, ctx_len,    \
                           tiles, n_tiles, decode_seqs, n_decode, max_decode_ctx, max_tile_ctx, mean_tile_walk,  \
                           workspace, out, nq, nkv, page_size, num_pages, st, scale)
  switch (hd / 16) {
    SP_MFMA(1); SP_MFMA(2); SP_MFMA(3); SP_MFMA(4); SP_MFMA(5); SP_MFMA(6); SP_MFMA(8);
    default:
      return attention_mfma_wide_sigmoid(s, q, q_stride, k_pool, v_pool, block_tables, max_blocks, q_start, q_len, ctx_len, tiles,
                                         n_tiles, decode_seqs, n_decode, max_decode_ctx, max_tile_ctx, mean_tile_walk, workspace,
                                         out, nq, nkv, hd, page_size, num_pages, st, scale);
  }
#undef SP_MFMA
}

}  // namespace sprout
