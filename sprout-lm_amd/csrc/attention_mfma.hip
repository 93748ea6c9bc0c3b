// bfloat16 attention with softmax weights: the instantiations, the sizes the kernels take, and the one-query kernel with the
// output projection folded in.
#include "attention_mfma.h"

namespace sprout {

bool attention_mfma_supports(int hd, int page_size, int nq, int nkv) {
  const int dt = hd / 16;
  const bool hd_ok = hd % 16 == 0 && (dt <= 6 || dt == 8 || dt == 10 || dt == 12 || dt == 16);
  return hd_ok && page_size % 4 == 0;
}
bool attention_mfma_decode_supports(int nq, int nkv) { return true; }
int attention_mfma_tile_q(int hd) { return 32; }

int attention_prefill_splits(int n_tiles, int nq, int nkv, int hd, int page_size, int max_tile_ctx) {
  if (!staged_prefill(page_size)) return 1;
  const StagedShape shape = staged_shape(nq, nkv, hd, n_tiles);
  const int G = nq / nkv;
  const int blocks = n_tiles * nkv * ((G + shape.hpb - 1) / shape.hpb), stages = (max_tile_ctx + kStageKeys - 1) / kStageKeys;
  const int enough = 2048 / (shape.wpt * shape.hpb);   // blocks that hold 2,048 waves: two rounds of the chip's CUs
  if (blocks <= 0 || blocks >= enough || stages <= 4) return 1;
  return max(1, min(min((enough * 3 / 2 + blocks - 1) / blocks, stages / 2), kMaxPrefillSplits));
}

size_t attention_prefill_workspace_floats(int n_tiles, int nq, int nkv, int hd, int page_size, int max_tile_ctx) {
  const size_t splits = attention_prefill_splits(n_tiles, nq, nkv, hd, page_size, max_tile_ctx);
  return splits <= 1 ? 0 : size_t(n_tiles) * 32 * nq * splits * (hd + 2);
}

size_t attention_decode_workspace_floats(int n_decode, int nq, int hd, int max_ctx) {
  const size_t splits = (max_ctx + kDecodeChunk - 1) / kDecodeChunk;
  return splits <= 1 ? 0 : size_t(n_decode) * nq * splits * (hd + 2);
}

int attention_mfma_wide(hipStream_t s, const void* q, int q_stride, const void* k_pool, const void* v_pool,
                        const int32_t* block_tables, int max_blocks, const int32_t* q_start, const int32_t* q_len,
                        const int32_t* ctx_len, const int32_t* tiles, int n_tiles, const int32_t* decode_seqs, int n_decode,
                        int max_decode_ctx, int max_tile_ctx, int mean_tile_walk, float* workspace, void* out, int nq, int nkv,
                        int hd, int page_size, int num_pages, ScoreStage st, float scale);

int attention_mfma(hipStream_t s, const void* q, int q_stride, const void* k_pool, const void* v_pool,
                   const int32_t* block_tables, int max_blocks, const int32_t* q_start, const int32_t* q_len,
                   const int32_t* ctx_len, const int32_t* tiles, int n_tiles, const int32_t* decode_seqs, int n_decode,
                   int max_decode_ctx, int max_tile_ctx, int mean_tile_walk, float* workspace, void* out, int nq, int nkv,
                   int hd, int page_size, int num_pages, ScoreStage st, float scale) {
#define SP_MFMA(DT)                                                                                              \
  case DT:                                                                                                       \
    return launch_mfma<DT, false>(s, q, q_stride, k_pool, v_pool, block_tables, max_blocks, q_start, q_len, ctx_len,    \
                           tiles, n_tiles, decode_seqs, n_decode, max_decode_ctx, max_tile_ctx, mean_tile_walk,  \
                           workspace, out, nq, nkv, page_size, num_pages, st, scale)
  switch (hd / 16) {
    SP_MFMA(1); SP_MFMA(2); SP_MFMA(3); SP_MFMA(4); SP_MFMA(5); SP_MFMA(6); SP_MFMA(8);
    default:
      return attention_mfma_wide(s, q, q_stride, k_pool, v_pool, block_tables, max_blocks, q_start, q_len, ctx_len, tiles, n_tiles,
                                 decode_seqs, n_decode, max_decode_ctx, max_tile_ctx, mean_tile_walk, workspace, out, nq, nkv, hd,
                                 page_size, num_pages, st, scale);
  }
#undef SP_MFMA
}

// Decode steps whose chunks' merge is folded into the output projection.  Worth it where the merged partial
// results, which every block of a head and a tile of 16 sequences reads again, stay small beside the rows of w_o
// (measured at 14 heads of 64, a width of 896, contexts of 4,096, tokens a second with the fold against merge and
// projection kernels of their own: 8 sequences 8,250 against 7,930, 24 sequences 21,870 against 21,260, 32
// sequences 27,400 against 26,660, 64 sequences 39,840 against 40,350).
bool attention_decode_project_takes(int hd, int page_size, int nq, int nkv, int n_decode, int max_decode_ctx, int hidden) {
  if (hd > 128 || !attention_mfma_supports(hd, page_size, nq, nkv) || !attention_mfma_decode_supports(nq, nkv)) return false;
  const int n_splits = (max_decode_ctx + kDecodeChunk - 1) / kDecodeChunk;
  return n_decode >= 1 && n_decode <= 32 && n_splits > 1 && min(n_decode, 16) * n_splits <= 256 && hidden >= 16 &&
         hidden <= 2048;   // (wider: 28 heads of 128 at 3,584 +1%, 40 heads at 5,120 -0.5% with four tiles a wave)
}

// Tiles of 16 rows of w_o a wave takes in the folded kernel: one up to 16 sequences; with more, every tile of 16
// sequences is a block of its own and merges the head's chunks again, so a block takes as many rows as still
// leaves about 200 blocks (24 and 32 sequences, 14 heads, a width of 896: two tiles a wave 21,870 and 27,400
// tokens a second, one 21,600 and 27,100, four 21,400 and 26,990).
static int project_tiles_per_wave(int n_decode, int nq, int hidden) {
  if (n_decode <= 16) return 1;
  const int seq_tiles = (n_decode + 15) / 16;
  for (int tpw = 4; tpw > 1; tpw /= 2)
    if (nq * ((hidden + 64 * tpw - 1) / (64 * tpw)) * seq_tiles >= 192) return tpw;
  return 1;
}

template <int DT>
static int launch_decode_project(hipStream_t s, const void* q, int q_stride, const void* k_pool, const void* v_pool,
                                 const int32_t* block_tables, int max_blocks, const int32_t* q_start,
                                 const int32_t* ctx_len, const int32_t* decode_seqs, int n_decode, int max_decode_ctx,
                                 float* workspace, const void* w_o, float* residual, int hidden, int nq, int nkv,
                                 int page_size, int num_pages, ScoreStage st, float scale) {
  constexpr int HD = 16 * DT;
  const int n_splits = (max_decode_ctx + kDecodeChunk - 1) / kDecodeChunk;
  float* part_o = workspace;
  float* part_ml = workspace + size_t(n_decode) * nq * n_splits * HD;
  if ((page_size & (page_size - 1)) == 0)
    attention_decode_kernel<DT, true, false><<<dim3(n_splits, decode_sets(nq, nkv), n_decode), 256, 0, s>>>(
        (const uint16_t*)q, q_stride, (const uint16_t*)k_pool, (const uint16_t*)v_pool, block_tables, max_blocks, q_start,
        ctx_len, decode_seqs, nullptr, part_o, part_ml, n_splits, nq, decode_sets(nq, nkv), nkv, page_size, num_pages, st,
        scale * kLog2e);
  else
    attention_decode_kernel<DT, false, false><<<dim3(n_splits, decode_sets(nq, nkv), n_decode), 256, 0, s>>>(
        (const uint16_t*)q, q_stride, (const uint16_t*)k_pool, (const uint16_t*)v_pool, block_tables, max_blocks, q_start,
        ctx_len, decode_seqs, nullptr, part_o, part_ml, n_splits, nq, decode_sets(nq, nkv), nkv, page_size, num_pages, st,
        scale * kLog2e);
  if (check_launch("sp_attention_decode_project (decode)")) return 1;
  const int tpw = project_tiles_per_wave(n_decode, nq, hidden);
  const dim3 grid(nq, (hidden + 64 * tpw - 1) / (64 * tpw), (n_decode + 15) / 16);
#define SP_PROJECT(TPW)                                                                                         \
  attention_merge_project_kernel<DT, 1, TPW><<<grid, 256, 0, s>>>(part_o, part_ml, q_start, decode_seqs,        \
                                                                   (const uint16_t*)w_o, residual, n_decode,     \
                                                                   n_splits, nq, hidden)
  if (tpw == 1) SP_PROJECT(1);
  else if (tpw == 2) SP_PROJECT(2);
  else SP_PROJECT(4);
#undef SP_PROJECT
  return check_launch("sp_attention_decode_project (merge and projection)");
}

int attention_mfma_decode_project(hipStream_t s, const void* q, int q_stride, const void* k_pool, const void* v_pool,
                                  const int32_t* block_tables, int max_blocks, const int32_t* q_start,
                                  const int32_t* ctx_len, const int32_t* decode_seqs, int n_decode, int max_decode_ctx,
                                  float* workspace, const void* w_o, float* residual, int hidden, int nq, int nkv,
                                  int hd, int page_size, int num_pages, ScoreStage st, float scale) {
#define SP_MFMA(DT)                                                                                              \
  case DT:                                                                                                       \
    return launch_decode_project<DT>(s, q, q_stride, k_pool, v_pool, block_tables, max_blocks, q_start, ctx_len, \
                                     decode_seqs, n_decode, max_decode_ctx, workspace, w_o, residual, hidden,    \
                                     nq, nkv, page_size, num_pages, st, scale)
  switch (hd / 16) {
    SP_MFMA(1); SP_MFMA(2); SP_MFMA(3); SP_MFMA(4); SP_MFMA(5); SP_MFMA(6); SP_MFMA(8);
  }
#undef SP_MFMA
  set_error("sp_attention_decode_project: no matrix-core kernel for head size %d", hd);
  return 1;
}

}  // namespace sprout
