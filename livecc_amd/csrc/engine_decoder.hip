// Layer-list decoders on the engine (family LCC_FAMILY_DECODER): a token model whose layers are described one by one -- a latent-attention
// mixer with its sizes, optionally reading the cache of an earlier layer, and a gated feed-forward or none -- with both sublayers in
// parallel behind one Dynamic-Tanh norm and an fp32 residual.  Slots, token state, meta ring, sampler, prefill / decode entry points are the
// engine's (engine.hip, engine_llm.hip); this file is the launch sequence of the layers and what they need in memory.
//
// A layer is
// (decode steps of up to 16 rows fuse "in" with "ff", the norms with "query", and "out" with the residual and the next norm: decode_v2.hip)
//   in      [Wdq | Wdkv | Wg] h           one GEMM, fp32 slabs
//           norms -> query latent, c -> cache, gates          (latent_norm_append)
//   query   Wuq cq                                            GEMM
//   attend  prefill: gather c, k = Uk c, v^T = Uv c^T (two GEMMs), multi-head attention       (attn_mha)
//           decode:  Uk^T q (latent_absorb), attention over c (latent_attn_decode), merge + Uv + gate (latent_merge_uv)
//   ff      silu(Wgate h) * (Wup h)       one GEMM, SwiGLU epilogue; lands beside the attention output
//   out     [Wo | Wdown] [attention | ff] one GEMM over the concatenated K: the sum of the parallel sublayers is its accumulator
//           residual += slabs; h = next norm                  (resid_dyt)
#include "engine_decoder.h"

namespace {

struct DecDims {       // maxima over the layers
  int W, in_n = 0, qp = 0, qd = 0, vd = 0, rp = 0, cat = 0, heads = 0; size_t hr = 0;
};
DecDims dims_of(const lcc_engine* e) {
  DecDims d; d.W = e->c.hidden_size;
  for (const lcc_decoder_layer& L : e->dl) {
    d.in_n = std::max(d.in_n, lcc_engine::dec_in_rows(L));
    d.qp = std::max(d.qp, L.q_rank_pad);
    d.qd = std::max(d.qd, L.heads * L.dim_pad);
    d.vd = std::max(d.vd, L.heads * L.vdim_pad);
    d.rp = std::max(d.rp, L.kv_rank_pad);
    d.cat = std::max(d.cat, L.heads * L.vdim_pad + L.ff_pad);
    d.heads = std::max(d.heads, L.heads);
    d.hr = std::max(d.hr, (size_t)L.heads * L.kv_rank_pad);
  }
  return d;
}
// rows of freshly formed keys one attention launch can hold: any single stream, or a whole call of fresh streams (each rounded up to 32)
size_t key_rows(const lcc_engine* e) { return std::max<size_t>(e->lim.max_kv_len, (size_t)e->lim.max_new_rows + 32 * (size_t)std::min(e->lim.max_slots, e->lim.max_new_rows)); }
}  // namespace
int decoder_logit_rows_max(const lcc_engine* e) { return std::max(std::min(256, e->lim.max_new_rows), std::min(e->lim.max_slots, LCC_MAX_DECODE_BATCH)); }
namespace {
// key splits of the decode attention for `rows` rows: two or more 64-key tiles per block once the chip is full
int decode_splits(const lcc_engine* e, int rows, int max_len) {
  static const int forced = [] { const char* v = getenv("LCC_LATENT_SPLITS"); return v ? atoi(v) : 0; }();
  const int ntile = (max_len + 63) / 64;
  if (forced > 0) return std::max(1, std::min(std::min(forced, LATENT_MAX_SPLIT), ntile));
  const int want = std::max(1, e->cu_count / std::max(1, rows));
  return std::max(1, std::min(std::min(want, ntile >= 256 ? LATENT_MAX_SPLIT : 64), ntile));      // (past 64 the merge costs what a tile saves, except on long caches)
}
size_t decode_slots(const lcc_engine* e) {     // (row, split) pairs of one decode launch, per head
  const int B = std::min(e->lim.max_slots, LCC_MAX_DECODE_BATCH);
  size_t n = 0;
  for (int b = 1; b <= B; ++b) n = std::max(n, (size_t)b * decode_splits(e, b, e->lim.max_kv_len));
  return n;
}
size_t carve(const lcc_engine* e, DecBuffers* b, char* base) {
  if (e->dc.block == LCC_BLOCK_SANDWICH) {
    Carver cv; cv.base = base;
    carve_mixers(e, b, cv);
    return cv.off + 4096;
  }
  const DecDims d = dims_of(e);
  const size_t S = std::max(e->lim.max_new_rows, std::min(e->lim.max_slots, LCC_MAX_DECODE_BATCH)), T = key_rows(e), V = e->c.vocab_size, LR = decoder_logit_rows_max(e);
  Carver cv; cv.base = base;
  b->x = cv.take<float>(S * d.W); b->h = cv.take<bf16_t>(S * d.W);
  const size_t nmax = std::max(std::max(d.in_n, d.qd), d.W);
  b->part_cap = std::max(std::max(S * nmax, (size_t)8 * 64 * nmax + 64), std::max(LR * V, (size_t)16 << 20));
  b->part = cv.take<float>(b->part_cap);
  b->gate = cv.take<float>(S * d.heads);
  b->cq = cv.take<bf16_t>(S * d.qp); b->q = cv.take<bf16_t>(S * d.qd); b->cat = cv.take<bf16_t>(S * d.cat);
  b->crow = cv.take<bf16_t>(T * d.rp); b->cfrag = cv.take<bf16_t>(T * d.rp);
  b->kmat = cv.take<bf16_t>(T * d.qd); b->vmat = cv.take<bf16_t>(T * d.vd);
  b->lat_q = cv.take<bf16_t>((size_t)LCC_MAX_DECODE_BATCH * d.hr);
  const size_t pairs = decode_slots(e);
  b->ws_o = cv.take<float>(pairs * d.hr); b->ws_ml = cv.take<float>(std::max(pairs * d.heads * 2, (size_t)LCC_MAX_DECODE_BATCH * 1024));
  b->last = cv.take<bf16_t>(LR * d.W);
  b->logits = cv.take<float>(LR * V);
  return cv.off + 4096;
}
int carve_bound(lcc_engine* e, DecBuffers* b) {
  if (carve(e, b, e->ws) > e->ws_bytes) return fail(LCC_ERR_STATE, "workspace too small");
  return 0;
}

}  // namespace
int g_fused_decode = 1;      // lcc_debug_set_decoder_fused: decode steps of up to 16 rows run the fused launches (6 per layer instead of 9)

namespace {
// S packed rows through every layer; pt null: a decode step over the streams `d_slots`.  On exit b.h holds the final norm of the residual.
int run_decoder_layers(lcc_engine* e, const DecBuffers& b, int S, const PrefillTables* pt, const int32_t* d_slots, int nsplit_attn, const AttnDirect& direct,
                       hipStream_t st) {
  const bool fused = !pt && S <= 16 && g_fused_decode;
  const int W = e->c.hidden_size, NL = (int)e->dl.size();
  if (e->llm_over) return fail(LCC_ERR_STATE, "per-layer input overrides are not available for this model family");
  LCC_TRY(tap(e, b, 0, S, st));
  for (int l = 0; l < NL; ++l) {
    const lcc_decoder_layer& L = e->dl[l];
    const DecLayerW& w = e->dw[l];
    const bool own = L.kv_from < 0;
    const int owner = own ? l : L.kv_from, rp = L.kv_rank_pad, in_n = lcc_engine::dec_in_rows(L), ldcat = L.heads * L.vdim_pad + L.ff_pad;
    const size_t kv_off = e->dec_off[owner].kv;
    const float scale_log2e = L.scale * 1.4426950408889634f;
    int ns = 1;
    if (fused) {
      DgArgs gi, gs;
      gi.W = w.in_w; gi.M = S; gi.N = in_n; gi.K = W; gi.X = b.h; gi.ldx = W; gi.C32 = b.part; gi.ldc = in_n;
      gs.W = w.gate_up_w; gs.M = S; gs.N = 2 * L.ff_pad; gs.K = W; gs.X = b.h; gs.ldx = W; gs.C = b.cat + L.heads * L.vdim_pad; gs.ldc = ldcat;
      LCC_TRY(dgemv_in_swiglu(gi, gs, st));
    } else {
      LCC_TRY(slab_gemm(b, b.h, W, w.in_w, S, in_n, W, &ns, st));
    }
    LatentInArgs in; in.part = b.part; in.nsplit = ns; in.rows = S; in.ldn = in_n; in.qp = L.q_rank_pad; in.rp = own ? rp : 0; in.q_rank = L.q_rank;
    in.kv_rank = L.kv_rank; in.heads = L.heads; in.eps = e->dc.norm_eps; in.q_norm = w.q_norm; in.kv_norm = w.kv_norm; in.cq = b.cq; in.gate = b.gate;
    in.tok_stream = pt ? pt->tok_stream : d_slots; in.tok_pos = pt ? pt->tok_pos : nullptr; in.kv_len = e->d_kv_len; in.kv_base = e->d_kv_base; in.kv_off = kv_off;
    const bool fused_q = fused && dgemv_latent_q_ok(S, L.q_rank_pad);
    if (!fused_q) LCC_TRY(latent_norm_append(in, st));
    if (pt) {
      LCC_TRY(plain_gemm(b.cq, L.q_rank_pad, w.uq_w, b.q, L.heads * L.dim_pad, S, L.heads * L.dim_pad, L.q_rank_pad, LCC_EPI_NONE, st));
      for (const KeyGroup& kg : pt->groups) {
        const int T = kg.n_tiles * 16;
        LCC_TRY(latent_gather(e->d_kv_base, kv_off, rp, pt->tile_slot + kg.tile0, pt->tile_key0 + kg.tile0, pt->tile_nkeys + kg.tile0, kg.n_tiles, b.crow, b.cfrag, st));
        LCC_TRY(plain_gemm(b.crow, rp, w.uk_w, b.kmat, L.heads * L.dim_pad, T, L.heads * L.dim_pad, rp, LCC_EPI_NONE, st));
        LCC_TRY(plain_gemm(w.uv_w, rp, b.cfrag, b.vmat, T, L.heads * L.vdim_pad, T, rp, LCC_EPI_NONE, st));      // v^T: the latents are the "weights"
        MhaArgs a; a.q = b.q + (size_t)kg.row0 * L.heads * L.dim_pad; a.k = b.kmat; a.vt = b.vmat; a.ldv = T; a.gate = b.gate + (size_t)kg.row0 * L.heads;
        a.out = b.cat + (size_t)kg.row0 * ldcat; a.ldo = ldcat; a.grp_q0 = pt->grp_q0 + kg.grp0; a.grp_nq = pt->grp_nq + kg.grp0;
        a.grp_pos0 = pt->grp_pos0 + kg.grp0; a.grp_key0 = pt->grp_key0 + kg.grp0; a.n_groups = kg.n_grps; a.rows = kg.n_rows; a.heads = L.heads;
        a.dim = L.dim_pad; a.vdim = L.vdim_pad; a.scale_log2e = scale_log2e;
        LCC_TRY(attn_mha(a, st));
      }
    } else {
      float* q32 = b.part;
      if (fused_q) {
        q32 = b.part + align_up((size_t)S * in_n, 64);      // beside the input projection it reads
        DgArgs gq; gq.W = w.uq_w; gq.M = S; gq.N = L.heads * L.dim_pad; gq.K = L.q_rank_pad; gq.S32 = b.part; gq.lds32 = in_n; gq.rank = L.q_rank;
        gq.norm_w = w.q_norm; gq.eps = e->dc.norm_eps; gq.C32 = q32; gq.ldc = gq.N;
        LCC_TRY(dgemv_latent_q(gq, in, st));
        ns = 1;
      } else {
        LCC_TRY(slab_gemm(b, b.cq, L.q_rank_pad, w.uq_w, S, L.heads * L.dim_pad, L.q_rank_pad, &ns, st));
      }
      LCC_TRY(latent_absorb(q32, ns, S, L.heads, L.dim_pad, w.ukt_w, rp, b.lat_q, st));
      LatentDecodeArgs a; a.q = b.lat_q; a.rows = S; a.heads = L.heads; a.rp = rp; a.nsplit = nsplit_attn; a.scale_log2e = scale_log2e; a.slots = d_slots;
      a.kv_len = e->d_kv_len; a.kv_base = e->d_kv_base; a.kv_off = kv_off; a.ws_o = b.ws_o; a.ws_ml = b.ws_ml; a.direct = direct;
      LCC_TRY(latent_attn_decode(a, st));
      LCC_TRY(latent_merge_uv(a, w.uv_w, L.vdim_pad, b.gate, b.cat, ldcat, st));
    }
    if (!fused && L.ff_pad > 0) LCC_TRY(plain_gemm(b.h, W, w.gate_up_w, b.cat + L.heads * L.vdim_pad, ldcat, S, 2 * L.ff_pad, W, LCC_EPI_SWIGLU, st));
    const DytNorm& next = l + 1 < NL ? e->dw[l + 1].norm : e->dec_final_norm;
    if (fused) {
      DgArgs go; go.W = w.out_w; go.M = S; go.N = W; go.K = ldcat; go.X = b.cat; go.ldx = ldcat; go.X32 = b.x; go.C = b.h; go.dyt = next;
      LCC_TRY(dgemv_resid_dyt(go, st));
    } else {
      LCC_TRY(slab_gemm(b, b.cat, ldcat, w.out_w, S, W, ldcat, &ns, st));
      LCC_TRY(resid_dyt(b.x, b.part, ns, next, b.h, S, W, st));
    }
    LCC_TRY(tap(e, b, l + 1, S, st));
  }
  return 0;
}

// x and the first norm of the rows' tokens: prefill ids per row, decode (pt null) the slots' current tokens
int embed_rows(lcc_engine* e, const DecBuffers& b, const int32_t* ids, const int32_t* d_slots, const PrefillTables* pt, int S, hipStream_t st) {
  if (e->dc.block != LCC_BLOCK_SANDWICH) return embed_dyt(ids, d_slots, e->embed, e->dw[0].norm, b.x, b.h, S, e->c.hidden_size, st);
  BigramEmbed bg; bg.table = e->dec_bigram; bg.buckets = e->dc.bigram_buckets; bg.mul_prev = e->dc.bigram_mul_prev; bg.mul_cur = e->dc.bigram_mul_cur;
  return embed_bigram_rms(ids, pt ? pt->tok_stream : d_slots, pt ? pt->tok_pos : nullptr, pt ? pt->tok_row0 : nullptr, e->d_kv_len, e->d_prev_tok, e->embed, bg,
                          e->dw[0].norm1, e->dc.norm_eps, b.x, b.h, S, e->dc.width, e->c.hidden_size, st);
}
int run_layers_of(lcc_engine* e, const DecBuffers& b, int S, const PrefillTables* pt, const int32_t* d_slots, int nsplit_attn, const AttnDirect& direct, hipStream_t st) {
  return e->dc.block == LCC_BLOCK_SANDWICH ? run_mixer_layers(e, b, S, pt, d_slots, nsplit_attn, direct, st)
                                           : run_decoder_layers(e, b, S, pt, d_slots, nsplit_attn, direct, st);
}

// logits of n rows of normed activations; `out` (row pitch = padded vocabulary, -inf beyond it) and / or `dense` (row pitch = vocabulary)
int decoder_logits(lcc_engine* e, const DecBuffers& b, const bf16_t* rows, int n, float* out, float* dense, hipStream_t st) {
  const int V = e->c.vocab_size;
  int ns = 1;
  LCC_TRY(slab_gemm(b, rows, e->c.hidden_size, e->lm_head, n, V, e->c.hidden_size, &ns, st));
  return logits_cap(b.part, ns, n, V, e->dc.vocab_size, e->dc.block == LCC_BLOCK_SANDWICH ? e->dc.logit_scale : 1.f, e->dc.logit_softcap, out, dense, st);
}
int head_and_sample_decoder(lcc_engine* e, const DecBuffers& b, const bf16_t* rows, int B, const int32_t* d_slots, const lcc_sampling* sp, int step_index,
                            hipStream_t st) {
  const int LR = decoder_logit_rows_max(e);
  for (int r0 = 0; r0 < B; r0 += LR) {       // (a prefill call may start more streams than one logits block holds)
    const int n = std::min(LR, B - r0);
    float* dense = (sp && sp->logits_out) ? (float*)sp->logits_out + ((size_t)step_index * B + r0) * e->dc.vocab_size : nullptr;
    LCC_TRY(decoder_logits(e, b, rows + (size_t)r0 * e->c.hidden_size, n, b.logits, dense, st));
    lcc_sampling part;
    if (sp) { part = *sp; if (part.scores_out) part.scores_out += (size_t)r0 * e->c.vocab_size; }
    LCC_TRY(lcc_sample_rows(e, b.logits, true, n, B, r0, d_slots + r0, sp ? &part : nullptr, step_index, b.ws_ml, st));
  }
  return 0;
}
}  // namespace

int lcc_engine::dec_in_rows(const lcc_decoder_layer& L) { return L.q_rank_pad + (L.kv_from < 0 ? L.kv_rank_pad : 0) + (L.heads + 15) / 16 * 16; }
size_t lcc_decoder_ws_bytes(const lcc_engine* e) { DecBuffers b; return carve(e, &b, nullptr); }
size_t lcc_decoder_meta_bytes(const lcc_engine* e) {
  if (e->dc.block == LCC_BLOCK_SANDWICH) return mixers_meta_ints(e) * 4;
  const size_t S = e->lim.max_new_rows, B = e->lim.max_slots;
  const size_t tiles = (S + 32 * B) / 16 + (size_t)std::min<size_t>(B, S) * (e->lim.max_kv_len / 16 + 2);      // new rows plus everything cached
  return (4 * S + 3 * tiles + 4 * (S / MHA_GROUP_ROWS + B + 1) + 4 * B + 256) * 4;
}

extern "C" lcc_engine* lcc_engine_create_decoder(const lcc_decoder_config* cfg, const lcc_decoder_layer* layers, const lcc_engine_limits* lim) {
  if (!cfg || !layers || !lim) { fail(LCC_ERR_ARG, "null config"); return nullptr; }
  if (cfg->n_layers < 1 || cfg->vocab_size < 1 || cfg->vocab_pad < cfg->vocab_size || (cfg->vocab_pad & 63) || cfg->width_pad < 64 || (cfg->width_pad & 63)) {
    fail(LCC_ERR_SHAPE, "decoder: layers >= 1, padded vocabulary and width in multiples of 64"); return nullptr;
  }
  if (lim->max_kv_len < 64 || (lim->max_kv_len & 63) || lim->max_slots <= 0 || lim->max_slots > 16 * 1024 || lim->max_new_rows <= 0 || lim->max_history <= 0) {
    fail(LCC_ERR_SHAPE, "decoder: max_kv_len %% 64, max_slots, max_new_rows, max_history"); return nullptr;
  }
  if (cfg->block != LCC_BLOCK_PARALLEL && cfg->block != LCC_BLOCK_SANDWICH) { fail(LCC_ERR_ARG, "decoder: unknown block form %d", cfg->block); return nullptr; }
  for (int i = 0; i < cfg->n_layers && cfg->block == LCC_BLOCK_PARALLEL; ++i) {
    const lcc_decoder_layer& L = layers[i];
    if (L.mixer != LCC_MIXER_LATENT) { fail(LCC_ERR_ARG, "decoder layer %d: unknown mixer %d", i, L.mixer); return nullptr; }
    if (L.heads < 1 || L.heads > 65535 || L.q_rank < 1 || L.kv_rank < 1 || L.q_rank_pad < L.q_rank || L.kv_rank_pad < L.kv_rank || (L.q_rank_pad & 63) ||
        (L.kv_rank_pad & 63) || L.dim_pad < 64 || (L.dim_pad & 63) || L.dim_pad > 1024 || L.vdim_pad < 64 || (L.vdim_pad & 63) || L.vdim_pad > 1024 ||
        L.ff_pad < 0 || (L.ff_pad & 63)) {
      fail(LCC_ERR_SHAPE, "decoder layer %d: padded sizes are multiples of 64, head sizes at most 1024", i); return nullptr;
    }
    const int rt = L.kv_rank_pad / 64;
    if (!(rt <= 4 || rt == 6 || rt == 8 || rt == 12 || rt == 16)) { fail(LCC_ERR_SHAPE, "decoder layer %d: padded latent rank %d has no kernel", i, L.kv_rank_pad); return nullptr; }
    if (L.kv_from >= i || (L.kv_from >= 0 && (layers[L.kv_from].kv_from >= 0 || layers[L.kv_from].kv_rank != L.kv_rank || layers[L.kv_from].kv_rank_pad != L.kv_rank_pad))) {
      fail(LCC_ERR_ARG, "decoder layer %d: kv_from %d is not an earlier layer with a latent of the same rank", i, L.kv_from); return nullptr;
    }
  }
  lcc_engine* e = new lcc_engine();
  e->family = LCC_FAMILY_DECODER;
  e->c = lcc_model_config{}; e->dc = *cfg; e->lim = *lim; e->lim.max_patches = 0;
  e->c.vocab_size = cfg->vocab_pad; e->c.hidden_size = cfg->width_pad; e->c.n_layers = cfg->n_layers; e->c.rms_eps = cfg->norm_eps;
  e->qd = e->kvd = e->qkvd = e->E = 0; e->vit_hd = 0; e->words = cfg->vocab_pad / 32; e->lay = KvLayout{0, 0, lim->max_kv_len, 0};
  e->dl.assign(layers, layers + cfg->n_layers);
  e->dw.resize(cfg->n_layers); e->dec_off.assign(cfg->n_layers, DecOffsets());
  if (cfg->block == LCC_BLOCK_SANDWICH) {
    if (mixers_layout(e) != 0) { delete e; return nullptr; }
  } else {
    size_t off = 0;
    for (int i = 0; i < cfg->n_layers; ++i)
      if (layers[i].kv_from < 0) { e->dec_off[i].kv = off; off += align_up((size_t)lim->max_kv_len * layers[i].kv_rank_pad, 128); }
    e->dec_kv_total = off;
  }
  e->chain_epoch.assign(128, 0u);
  { int dev = 0; if (hipGetDevice(&dev) == hipSuccess) (void)hipDeviceGetAttribute(&e->cu_count, hipDeviceAttributeMultiprocessorCount, dev); }
  if (e->cu_count <= 0) e->cu_count = 256;
  e->h_kv_len.assign(lim->max_slots, 0); e->h_pos.assign(lim->max_slots, 0); e->h_kv_base.assign(lim->max_slots, nullptr);
  return e;
}

int lcc_decoder_resolve_weights(lcc_engine* e, std::string* missing) {
  if (e->dc.block == LCC_BLOCK_SANDWICH) return mixers_resolve_weights(e, missing);
  auto get = [&](const std::string& n) -> const bf16_t* {
    auto it = e->w.find(n);
    if (it == e->w.end()) { if (missing) { *missing += n; *missing += ' '; } return nullptr; }
    return (const bf16_t*)it->second;
  };
  auto norm = [&](const std::string& p) { DytNorm n; n.w = get(p + "_w"); n.b = get(p + "_b"); n.alpha = get(p + "_alpha"); return n; };
  e->embed = get("embed"); e->lm_head = get("lm_head"); e->dec_final_norm = norm("final_norm");
  for (size_t i = 0; i < e->dl.size(); ++i) {
    const lcc_decoder_layer& L = e->dl[i];
    const std::string p = "dec." + std::to_string(i) + ".";
    DecLayerW& w = e->dw[i];
    w.norm = norm(p + "norm");
    w.in_w = get(p + "in_w"); w.q_norm = get(p + "q_norm"); w.kv_norm = L.kv_from < 0 ? get(p + "kv_norm") : nullptr;
    w.uq_w = get(p + "uq_w"); w.uk_w = get(p + "uk_w"); w.ukt_w = get(p + "ukt_w"); w.uv_w = get(p + "uv_w"); w.out_w = get(p + "out_w");
    w.gate_up_w = L.ff_pad > 0 ? get(p + "gate_up_w") : nullptr;
  }
  return missing && !missing->empty() ? LCC_ERR_STATE : 0;
}

// lcc_llm_prefill behind its argument checks (engine_llm.hip): mutex held, capacities and ids checked, S = total rows
int lcc_decoder_prefill(lcc_engine* e, int n_streams, const int32_t* slots, const int32_t* n_new, const int32_t* ids, int S, const lcc_sampling* sp, hipStream_t st) {
  DecBuffers bf; LCC_TRY(carve_bound(e, &bf));
  const int nw = sp ? sp->n_prompt_rows : 0;
  for (int i = 0; i < nw; ++i)
    if (!sp->prompt_rows || !sp->prompt_logits_out || sp->prompt_rows[i] < 0 || sp->prompt_rows[i] >= S) return fail(LCC_ERR_ARG, "prompt_rows[%d] out of range", i);
  PrefillTables pt;
  std::vector<int32_t> tok_stream(S), tok_pos(S), last_row(n_streams), ts, tk, tn, gq, gn, gp, gk;
  const bool mixers = e->dc.block == LCC_BLOCK_SANDWICH;
  const size_t cap_tiles = mixers ? ~(size_t)0 : key_rows(e) / 16;
  std::vector<int32_t> row0, rlast, gs, sr, sn, ss, sf, st0, stn;
  const int seg = mixers ? mixers_segment_rows(e, bf, n_new, n_streams) : 0;
  int row = 0;
  KeyGroup kg{0, 0, 0, 0, 0, 0};
  for (int b = 0; b < n_streams; ++b) {
    const int past = e->h_kv_len[slots[b]], keys = past + n_new[b], tiles = mixers ? 0 : (keys + 31) / 32 * 2;
    if (kg.n_rows > 0 && (size_t)(kg.n_tiles + tiles) > cap_tiles) {
      pt.groups.push_back(kg);
      kg = KeyGroup{(int)ts.size(), 0, (int)gq.size(), 0, row, 0};
    }
    for (int i = 0; i < n_new[b]; ++i) { tok_stream[row + i] = slots[b]; tok_pos[row + i] = past + i; }
    for (int q = 0; q < n_new[b]; q += MHA_GROUP_ROWS) {       // rows and key rows relative to their key group
      gq.push_back(row - kg.row0 + q); gn.push_back(std::min(MHA_GROUP_ROWS, n_new[b] - q)); gp.push_back(past + q); gk.push_back(kg.n_tiles * 16);
    }
    for (int t = 0; t < tiles; ++t) { ts.push_back(slots[b]); tk.push_back(t * 16); tn.push_back(keys); }
    if (mixers) {
      st0.push_back((int)sr.size());
      for (int q = 0; q < n_new[b]; q += seg) { sr.push_back(row + q); sn.push_back(std::min(seg, n_new[b] - q)); ss.push_back(slots[b]); sf.push_back(past + q == 0); }
      stn.push_back((int)sr.size() - st0.back());
      for (int q = 0; q < n_new[b]; q += MHA_GROUP_ROWS) gs.push_back(slots[b]);
      for (int i = 0; i < n_new[b]; ++i) { row0.push_back(row); rlast.push_back(row + n_new[b] - 1); }
    }
    kg.n_tiles += tiles; kg.n_grps = (int)gq.size() - kg.grp0; kg.n_rows += n_new[b];
    row += n_new[b];
    last_row[b] = row - 1;
  }
  pt.groups.push_back(kg);
  MetaWriter mw; LCC_TRY(meta_begin(e, &mw));
  int32_t *d_ids, *d_stream, *d_pos, *d_last, *d_slots, *d_ts, *d_tk, *d_tn, *d_gq, *d_gn, *d_gp, *d_gk, *d_want = nullptr;
  bool ok = mw.put(ids, S, &d_ids) && mw.put(tok_stream.data(), S, &d_stream) && mw.put(tok_pos.data(), S, &d_pos) && mw.put(last_row.data(), n_streams, &d_last) &&
            mw.put(slots, n_streams, &d_slots) && mw.put(ts.data(), ts.size(), &d_ts) && mw.put(tk.data(), tk.size(), &d_tk) && mw.put(tn.data(), tn.size(), &d_tn) &&
            mw.put(gq.data(), gq.size(), &d_gq) && mw.put(gn.data(), gn.size(), &d_gn) && mw.put(gp.data(), gp.size(), &d_gp) && mw.put(gk.data(), gk.size(), &d_gk);
  int32_t *d_row0 = nullptr, *d_rlast = nullptr, *d_gs = nullptr, *d_sr = nullptr, *d_sn = nullptr, *d_ss = nullptr, *d_sf = nullptr, *d_st0 = nullptr, *d_stn = nullptr;
  if (ok && mixers)
    ok = mw.put(row0.data(), S, &d_row0) && mw.put(rlast.data(), S, &d_rlast) && mw.put(gs.data(), gs.size(), &d_gs) && mw.put(sr.data(), sr.size(), &d_sr) &&
         mw.put(sn.data(), sn.size(), &d_sn) && mw.put(ss.data(), ss.size(), &d_ss) && mw.put(sf.data(), sf.size(), &d_sf) &&
         mw.put(st0.data(), st0.size(), &d_st0) && mw.put(stn.data(), stn.size(), &d_stn);
  if (ok && nw > 0) ok = nw <= S && mw.put(sp->prompt_rows, nw, &d_want) != nullptr;
  if (!ok) return fail(LCC_ERR_STATE, "meta ring slot too small");
  LCC_TRY(meta_commit(&mw, st));
  pt.tok_stream = d_stream; pt.tok_pos = d_pos; pt.tile_slot = d_ts; pt.tile_key0 = d_tk; pt.tile_nkeys = d_tn;
  pt.grp_q0 = d_gq; pt.grp_nq = d_gn; pt.grp_pos0 = d_gp; pt.grp_key0 = d_gk;

  pt.tok_row0 = d_row0; pt.tok_last = d_rlast; pt.grp_slot = d_gs; pt.seg_row0 = d_sr; pt.seg_rows = d_sn; pt.seg_slot = d_ss; pt.seg_fresh = d_sf;
  pt.str_seg0 = d_st0; pt.str_nseg = d_stn; pt.n_grps = (int)gq.size(); pt.n_seg = (int)sr.size(); pt.n_streams = n_streams;

  for (int b = 0; b < n_streams; ++b) {      // a new generate call of these slots
    HIP_TRY(hipMemsetAsync(e->d_hist_col + slots[b], 0, 4, st));
    HIP_TRY(hipMemsetAsync(e->d_done + slots[b], 0, 4, st));
  }
  LCC_TRY(seen_set(e->d_seen, e->words, d_ids, d_stream, S, 0, nullptr, st));
  LCC_TRY(embed_rows(e, bf, d_ids, nullptr, &pt, S, st));
  LCC_TRY(run_layers_of(e, bf, S, &pt, nullptr, 1, AttnDirect(), st));

  const int LR = decoder_logit_rows_max(e), W = e->c.hidden_size;
  for (int r0 = 0; r0 < nw; r0 += LR) {
    const int n = std::min(LR, nw - r0);
    LCC_TRY(gather_rows_bf16(bf.h, d_want + r0, bf.last, n, W, st));
    LCC_TRY(decoder_logits(e, bf, bf.last, n, nullptr, sp->prompt_logits_out + (size_t)r0 * e->dc.vocab_size, st));
  }
  std::vector<int32_t> kv(n_streams);
  for (int b = 0; b < n_streams; ++b) { e->h_kv_len[slots[b]] += n_new[b]; e->h_pos[slots[b]] = kv[b] = e->h_kv_len[slots[b]]; }
  MetaWriter mw2; LCC_TRY(meta_begin(e, &mw2));
  int32_t* d_kv;
  if (!mw2.put(kv.data(), n_streams, &d_kv)) return fail(LCC_ERR_STATE, "meta ring slot too small");
  LCC_TRY(meta_commit(&mw2, st));
  for (int b = 0; b < n_streams; ++b) {
    HIP_TRY(hipMemcpyAsync(e->d_kv_len + slots[b], d_kv + b, 4, hipMemcpyDeviceToDevice, st));
    HIP_TRY(hipMemcpyAsync(e->d_pos + slots[b], d_kv + b, 4, hipMemcpyDeviceToDevice, st));
    HIP_TRY(hipMemcpyAsync(e->d_prev_tok + slots[b], d_ids + last_row[b], 4, hipMemcpyDeviceToDevice, st));
  }
  // the streams' last rows: gathered in blocks the logits buffer holds
  for (int r0 = 0; r0 < n_streams; r0 += LR) {
    const int n = std::min(LR, n_streams - r0);
    LCC_TRY(gather_rows_bf16(bf.h, d_last + r0, bf.last, n, W, st));
    float* dense = (sp && sp->logits_out) ? (float*)sp->logits_out + (size_t)r0 * e->dc.vocab_size : nullptr;
    lcc_sampling part;
    if (sp) { part = *sp; part.logits_out = dense; if (part.scores_out) part.scores_out += (size_t)r0 * e->c.vocab_size; }
    LCC_TRY(decoder_logits(e, bf, bf.last, n, bf.logits, dense, st));
    LCC_TRY(lcc_sample_rows(e, bf.logits, true, n, n_streams, r0, d_slots + r0, sp ? &part : nullptr, 0, bf.ws_ml, st));
  }
  return check_launch("lcc_llm_prefill");
}

// the n_steps loop of lcc_llm_decode (engine_llm.hip) behind its checks
int lcc_decoder_decode(lcc_engine* e, int n_streams, const int32_t* slots, const int32_t* d_slots, int max_len, int n_steps, int first_step_index, const lcc_sampling* sp, hipStream_t st) {
  DecBuffers bf; LCC_TRY(carve_bound(e, &bf));
  const int nsplit = e->dc.block == LCC_BLOCK_SANDWICH ? mixers_decode_splits(e, n_streams, max_len) : decode_splits(e, n_streams, max_len);
  for (int step = 0; step < n_steps; ++step) {
    const bool prof_step = e->prof_on && (step & 3) == 0 && 2 * (e->step_n + 1) <= (int)e->step_ev.size();
    if (prof_step) HIP_TRY(hipEventRecord(e->step_ev[2 * e->step_n], st));
    LCC_TRY(seen_set(e->d_seen, e->words, e->d_cur_tok, d_slots, n_streams, 1, e->d_done, st));
    LCC_TRY(embed_rows(e, bf, e->d_cur_tok, d_slots, nullptr, n_streams, st));
    AttnDirect dir;      // (a stream that EOS froze on the device has fewer keys than the host counts: its step is discarded, and the rows exist)
    if (n_streams <= 4) {
      for (int b = 0; b < n_streams; ++b) { dir.base[b] = (const bf16_t*)e->h_kv_base[slots[b]]; dir.n[b] = e->h_kv_len[slots[b]] + step + 1; }
      dir.used = n_streams;
    }
    LCC_TRY(run_layers_of(e, bf, n_streams, nullptr, d_slots, nsplit, dir, st));
    LCC_TRY(advance_lengths(d_slots, e->d_kv_len, e->d_pos, n_streams, e->d_done, st, e->d_cur_tok, e->d_prev_tok));
    LCC_TRY(head_and_sample_decoder(e, bf, bf.h, n_streams, d_slots, sp, first_step_index + step, st));
    if (prof_step) {
      HIP_TRY(hipEventRecord(e->step_ev[2 * e->step_n + 1], st));
      if (e->step_n < (int)e->step_rel.size()) e->step_rel[e->step_n] = step;
      e->step_n++;
    }
  }
  return check_launch("lcc_llm_decode");
}

extern "C" int lcc_slot_set_tokens(lcc_engine* e, int n_streams, const int32_t* slots, const int32_t* tokens, void* stream) {
  if (!e || n_streams <= 0 || n_streams > e->lim.max_slots || !slots || !tokens) return fail(LCC_ERR_ARG, "bad argument");
  if (!e->state) return fail(LCC_ERR_STATE, "buffers not bound");
  std::lock_guard<std::mutex> lk(e->mu_llm);
  const int vocab = e->family == LCC_FAMILY_DECODER ? e->dc.vocab_size : e->c.vocab_size;
  for (int b = 0; b < n_streams; ++b) {
    if (slots[b] < 0 || slots[b] >= e->lim.max_slots) return fail(LCC_ERR_ARG, "bad slot %d", slots[b]);
    if (tokens[b] < 0 || tokens[b] >= vocab) return fail(LCC_ERR_ARG, "token id %d out of range", tokens[b]);
  }
  MetaWriter mw; LCC_TRY(meta_begin(e, &mw));
  int32_t *d_slots, *d_tok;
  if (!mw.put(slots, n_streams, &d_slots) || !mw.put(tokens, n_streams, &d_tok)) return fail(LCC_ERR_STATE, "meta ring slot too small");
  LCC_TRY(meta_commit(&mw, (hipStream_t)stream));
  LCC_TRY(set_tokens(d_slots, d_tok, n_streams, e->d_cur_tok, e->d_done, e->d_hist_col, (hipStream_t)stream));
  return check_launch("lcc_slot_set_tokens");
}
extern "C" int lcc_debug_set_decoder_fused(int on) {
  if (lcc_knob_guard("lcc_debug_set_decoder_fused")) return -1;
  const int old = g_fused_decode;
  g_fused_decode = on ? 1 : 0;
  return old;
}
