// bfloat16 attention with sigmoid weights, head sizes above 128.  The kernels of attention_mfma.h, instantiated in a file of their own so that they compile beside the others.
#include "attention_mfma.h"

namespace sprout {

int attention_mfma_wide_sigmoid(hipStream_t s, const void* q, int q_stride, const void* k_pool, const void* v_pool,
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
    SP_MFMA(10); SP_MFMA(12); SP_MFMA(16);
  }
#undef SP_MFMA
  set_error("sp_attention: no matrix-core kernel for head size %d", hd);
  return 1;
}

}  // namespace sprout
