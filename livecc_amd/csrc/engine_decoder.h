// Shared by the two launch sequences of the layer-list decoders: engine_decoder.hip (entry points, parallel sublayers) and engine_mixers.hip
// (sequential sublayers with norms on both sides).
#pragma once
#include "engine_internal.h"

struct DecBuffers {
  float *x, *part, *gate, *ws_o, *ws_ml, *logits;
  bf16_t *h, *cq, *q, *cat, *kmat, *vmat, *crow, *cfrag, *lat_q, *last;
  size_t part_cap;     // floats
  // LCC_BLOCK_SANDWICH
  bf16_t *rq, *rk, *rv, *att, *rec, *act;
  float *dt, *y, *seg_state, *seg_decay;
  int seg_cap;
};
struct KeyGroup {       // streams whose keys are formed together
  int tile0, n_tiles, grp0, n_grps, row0, n_rows;
};
struct PrefillTables {
  const int32_t *tok_stream, *tok_pos, *tile_slot, *tile_key0, *tile_nkeys, *grp_q0, *grp_nq, *grp_pos0, *grp_key0;
  std::vector<KeyGroup> groups;
  // LCC_BLOCK_SANDWICH
  const int32_t *tok_row0 = nullptr, *tok_last = nullptr, *grp_slot = nullptr, *seg_row0 = nullptr, *seg_rows = nullptr, *seg_slot = nullptr, *seg_fresh = nullptr,
                *str_seg0 = nullptr, *str_nseg = nullptr;
  int n_grps = 0, n_seg = 0, n_streams = 0;
};

// rows of logits the workspace holds at once
int decoder_logit_rows_max(const lcc_engine* e);
extern int g_fused_decode;      // lcc_debug_set_decoder_fused
// fp32 slab product into `out` (null: b.part) of `cap` floats; the split count is the one the tiles or the weight-streaming kernels want, bounded by the slab buffer
static inline int slab_gemm(const DecBuffers& b, const bf16_t* A, int lda, const bf16_t* W, int M, int N, int K, int* nsplit, hipStream_t st, float* out = nullptr, size_t cap = 0) {
  if (!out) { out = b.part; cap = b.part_cap; }
  int s = gemm_routes_skinny(M, K, false) ? gemv_num_splits(N, K) : gemm_tiled_num_splits(M, N, K, true);
  s = std::min(std::min(s, 8), (K + 63) / 64);
  while (s > 1 && (size_t)s * M * N > cap) --s;
  if ((size_t)s * M * N > cap) return fail(LCC_ERR_STATE, "slab buffer too small for %d x %d", M, N);
  GemmArgs g; g.A = A; g.lda = lda; g.W = W; g.ldw = K; g.w_packed = 1; g.M = M; g.N = N; g.K = K; g.partial = out; g.nsplit = s;
  *nsplit = s;
  return gemm_bf16(g, st);
}
static inline int plain_gemm(const bf16_t* A, int lda, const bf16_t* W, bf16_t* C, int ldc, int M, int N, int K, int epilogue, hipStream_t st) {
  GemmArgs g; g.A = A; g.lda = lda; g.W = W; g.ldw = K; g.w_packed = 1; g.C = C; g.ldc = ldc; g.M = M; g.N = N; g.K = K; g.epilogue = epilogue;
  return gemm_bf16(g, st);
}

static inline int tap(lcc_engine* e, const DecBuffers& b, int index, int S, hipStream_t st) {
  if (!e->llm_taps) return 0;
  if (S > e->llm_tap_rows) return fail(LCC_ERR_STATE, "taps bound for %d rows, call has %d", e->llm_tap_rows, S);
  const size_t W = e->c.hidden_size;
  HIP_TRY(hipMemcpyAsync((float*)e->llm_taps + (size_t)index * e->llm_tap_rows * W, b.x, (size_t)S * W * 4, hipMemcpyDeviceToDevice, st));
  return 0;
}

// engine_mixers.hip
void carve_mixers(const lcc_engine* e, DecBuffers* b, Carver& cv);
size_t mixers_meta_ints(const lcc_engine* e);
int mixers_layout(lcc_engine* e);                        // dec_off, dec_kv_total; an error when a size has no kernel
int mixers_resolve_weights(lcc_engine* e, std::string* missing);
int mixers_segment_rows(const lcc_engine* e, const DecBuffers& b, const int32_t* n_new, int n_streams);
int mixers_decode_splits(const lcc_engine* e, int rows, int max_len);
int run_mixer_layers(lcc_engine* e, const DecBuffers& b, int S, const PrefillTables* pt, const int32_t* d_slots, int nsplit_attn, const AttnDirect& direct, hipStream_t st);
