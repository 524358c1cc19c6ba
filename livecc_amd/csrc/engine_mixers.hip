// Layer-list decoders whose sublayers run one after the other with an RMS norm before and after each (LCC_BLOCK_SANDWICH): grouped-query attention with a
// distance bias beside linear attention (LCC_MIXER_PARALLEL), state-space layers (LCC_MIXER_SSD), SwiGLU feed-forwards.  Entry points, embedding and
// logits: engine_decoder.hip.  A layer is
//   in      every projection of the mixer                 one product, fp32
//   prefill prep (norms, temperature, cache append | convolution, activations)      mixer_prep
//           attention (attn_mha over the slots' arenas), recurrence (rec_scan), gated norm (rec_norm)
//   decode  recurrence with its input activations and the attention's splits        rec_gqa_decode (other sizes, many rows: rec_decode, gqa_decode)
//           merge + gated norm in one launch                                        gqa_merge_rec_norm
//   out     W_o of the attention and of the recurrence    two products (decode: one launch), fp32
//           norms, residual, next norm                    post_norm_resid
//   ff      SwiGLU product, down product, post_norm_resid
// A slot's arena: per layer K and V (attention), the fp32 state of the recurrence, the last inputs of its convolution.
#include "engine_decoder.h"

namespace {
int up64(int n) { return (n + 63) / 64 * 64; }
int rec_inner(const lcc_decoder_layer& L) { return up64(L.rec_heads * L.rec_vdim); }
bool has_attn(const lcc_decoder_layer& L) { return L.mixer == LCC_MIXER_PARALLEL; }
int attn_cols(const lcc_decoder_layer& L) { return has_attn(L) ? (L.heads + L.kv_heads) * L.dim_pad + L.kv_heads * L.vdim_pad : 0; }
int conv_channels(const lcc_decoder_layer& L) { return L.rec_heads * L.rec_vdim_pad + 2 * L.rec_groups * L.rec_key_pad; }
int in_rows(const lcc_decoder_layer& L) {
  const int hv = L.rec_heads * L.rec_vdim_pad;
  return attn_cols(L) + hv + conv_channels(L) + (L.mixer == LCC_MIXER_SSD ? up64(L.rec_heads) : 0);
}
// columns of the recurrent part: parallel q | k | v | gate, state-space z | x | B | C | dt
RecInArgs rec_cols(const lcc_decoder_layer& L) {
  RecInArgs r;
  const int hv = L.rec_heads * L.rec_vdim_pad, gk = L.rec_groups * L.rec_key_pad, c0 = attn_cols(L);
  r.heads = L.rec_heads; r.groups = L.rec_groups; r.np = L.rec_key_pad; r.ep = L.rec_vdim_pad; r.ldn = in_rows(L);
  if (L.mixer == LCC_MIXER_SSD) {
    r.v_col = hv; r.k_col = 2 * hv; r.q_col = 2 * hv + gk; r.dt_col = 2 * hv + 2 * gk;
    r.taps = L.rec_conv_taps; r.conv_col = hv; r.conv_ch = conv_channels(L);
  } else {
    r.q_col = c0; r.k_col = c0 + gk; r.v_col = c0 + 2 * gk;
  }
  return r;
}
int gate_col(const lcc_decoder_layer& L) { return L.mixer == LCC_MIXER_SSD ? 0 : attn_cols(L) + 2 * L.rec_groups * L.rec_key_pad + L.rec_heads * L.rec_vdim_pad; }

struct Dims { size_t in_n = 0, q = 0, att = 0, gk = 0, hv = 0, rin = 0, ff = 0, heads = 0, rh = 0, state = 0; };
Dims dims_of(const lcc_engine* e) {
  Dims d;
  auto up = [](size_t& a, size_t b) { a = std::max(a, b); };
  for (const lcc_decoder_layer& L : e->dl) {
    up(d.in_n, in_rows(L)); up(d.gk, (size_t)L.rec_groups * L.rec_key_pad); up(d.hv, (size_t)L.rec_heads * L.rec_vdim_pad); up(d.rin, rec_inner(L));
    up(d.ff, L.ff_pad); up(d.rh, L.rec_heads); up(d.state, (size_t)L.rec_heads * L.rec_key_pad * L.rec_vdim_pad);
    if (has_attn(L)) { up(d.q, (size_t)L.heads * L.dim_pad); up(d.att, (size_t)L.heads * L.vdim_pad); up(d.heads, L.heads); }
  }
  return d;
}
size_t max_rows(const lcc_engine* e) { return std::max(e->lim.max_new_rows, std::min(e->lim.max_slots, LCC_MAX_DECODE_BATCH)); }
int max_batch(const lcc_engine* e) { return std::min(e->lim.max_slots, LCC_MAX_DECODE_BATCH); }
constexpr int SEG_CHUNKS = 4;          // shortest segment of the recurrence, in 64-token chunks
}  // namespace

int mixers_decode_splits(const lcc_engine* e, int rows, int max_len) {
  int kvh = 1;
  for (const lcc_decoder_layer& L : e->dl) if (has_attn(L)) kvh = std::max(kvh, L.kv_heads * ((L.heads / L.kv_heads + 15) / 16));
  const int ntile = (max_len + 31) / 32, want = std::max(1, 4 * e->cu_count / std::max(1, rows * kvh));      // one-wave blocks
  return std::max(1, std::min(std::min(want, (ntile + 1) / 2), GQA_MAX_SPLIT));
}

void carve_mixers(const lcc_engine* e, DecBuffers* b, Carver& cv) {
  const Dims d = dims_of(e);
  const size_t S = max_rows(e), W = e->c.hidden_size, V = e->c.vocab_size, LR = decoder_logit_rows_max(e), B = max_batch(e);
  *b = DecBuffers{};
  b->x = cv.take<float>(S * W); b->h = cv.take<bf16_t>(S * W);
  const size_t nmax = std::max(d.in_n, 2 * W);
  b->part_cap = std::max(std::max(S * nmax, (size_t)8 * 64 * nmax + 64), std::max(LR * V, (size_t)16 << 20));
  b->part = cv.take<float>(b->part_cap);
  b->q = cv.take<bf16_t>(S * d.q); b->att = cv.take<bf16_t>(S * d.att);
  b->rq = cv.take<bf16_t>(S * d.gk); b->rk = cv.take<bf16_t>(S * d.gk); b->rv = cv.take<bf16_t>(S * d.hv); b->dt = cv.take<float>(S * d.rh);
  b->y = cv.take<float>(S * d.hv); b->rec = cv.take<bf16_t>(S * d.rin); b->act = cv.take<bf16_t>(S * d.ff);
  b->seg_cap = (int)(S / (REC_CHUNK * SEG_CHUNKS) + std::min<size_t>(e->lim.max_slots, S) + 1);
  if (S <= (size_t)2 * REC_CHUNK * SEG_CHUNKS) b->seg_cap = 0;      // never cut into segments
  b->seg_state = cv.take<float>((size_t)b->seg_cap * d.state); b->seg_decay = cv.take<float>((size_t)b->seg_cap * d.rh);
  size_t pairs = 1;
  for (size_t r = 1; r <= B; ++r) pairs = std::max(pairs, r * mixers_decode_splits(e, (int)r, e->lim.max_kv_len));
  size_t vd = 64;
  for (const lcc_decoder_layer& L : e->dl) if (has_attn(L)) vd = std::max(vd, (size_t)L.vdim_pad);
  b->ws_o = cv.take<float>(pairs * d.heads * vd); b->ws_ml = cv.take<float>(std::max(pairs * d.heads * 2, (size_t)LCC_MAX_DECODE_BATCH * 1024));
  b->last = cv.take<bf16_t>(LR * W);
  b->logits = cv.take<float>(LR * V);
}
size_t mixers_meta_ints(const lcc_engine* e) {
  const size_t S = e->lim.max_new_rows, B = std::min(e->lim.max_slots, e->lim.max_new_rows);
  return 7 * S + 5 * (S / MHA_GROUP_ROWS + B + 1) + 4 * (S / REC_CHUNK + B + 1) + 6 * (size_t)e->lim.max_slots + 512;
}
// rows per segment of the recurrence: whole streams while they are short (one launch instead of three), else enough segments to fill the chip
int mixers_segment_rows(const lcc_engine* e, const DecBuffers& b, const int32_t* n_new, int n_streams) {
  int longest = 0;
  for (int i = 0; i < n_streams; ++i) longest = std::max(longest, n_new[i]);
  if (longest <= 2 * SEG_CHUNKS * REC_CHUNK || b.seg_cap == 0) return std::max(longest, 1);
  // time of a segment length = rounds of blocks on the chip (two resident per compute unit) x chunks per block, plus about one chunk per block to
  // start and to pass a state on; the layer with the most (head, 64 value channels) pairs decides
  long blocks = 1;
  for (const lcc_decoder_layer& L : e->dl) blocks = std::max(blocks, (long)L.rec_heads * (L.rec_vdim_pad / 64));
  long per = SEG_CHUNKS, best = -1;
  for (long c = SEG_CHUNKS; c <= 64; ++c) {
    long segs = 0;
    for (int i = 0; i < n_streams; ++i) segs += (n_new[i] + c * REC_CHUNK - 1) / (c * REC_CHUNK);
    const long cost = ((segs * blocks + 2 * e->cu_count - 1) / (2 * e->cu_count)) * (c + 1);
    if (best < 0 || cost < best) { best = cost; per = c; }
  }
  return (int)std::min<long>(per * REC_CHUNK, std::max(longest, 1));
}

int mixers_layout(lcc_engine* e) {
  const lcc_decoder_config& c = e->dc;
  if (c.width < 1 || c.width > c.width_pad || c.width_pad > 8192 || c.bigram_buckets < 1 || c.bigram_mul_prev < 0 || c.bigram_mul_cur < 0)
    return fail(LCC_ERR_SHAPE, "decoder: width in 1..width_pad <= 8192, bigram buckets >= 1");
  size_t off = 0;
  const size_t Lmax = e->lim.max_kv_len;
  for (size_t i = 0; i < e->dl.size(); ++i) {
    const lcc_decoder_layer& L = e->dl[i];
    DecOffsets& o = e->dec_off[i];
    if (L.mixer != LCC_MIXER_PARALLEL && L.mixer != LCC_MIXER_SSD) return fail(LCC_ERR_ARG, "decoder layer %d: unknown mixer %d", (int)i, L.mixer);
    if (L.rec_heads < 1 || L.rec_groups < 1 || L.rec_heads % L.rec_groups || L.rec_key_pad < 64 || (L.rec_key_pad & 63) || L.rec_key_pad > 256 || L.rec_vdim < 1 ||
        L.rec_vdim_pad < L.rec_vdim || (L.rec_vdim_pad & 63) || L.rec_norm_groups < 1 || (L.rec_heads * L.rec_vdim) % L.rec_norm_groups || L.ff_pad < 0 || (L.ff_pad & 63) ||
        (long)L.rec_heads * (L.rec_vdim_pad / 64) > 65535)
      return fail(LCC_ERR_SHAPE, "decoder layer %d: recurrent sizes", (int)i);
    if (L.mixer == LCC_MIXER_SSD ? L.rec_conv_taps < 1 || L.rec_conv_taps > 16 : L.rec_conv_taps != 0 || L.rec_groups != L.rec_heads)
      return fail(LCC_ERR_SHAPE, "decoder layer %d: convolution taps", (int)i);
    if (has_attn(L)) {
      if (L.heads < 1 || L.heads > 65535 || L.kv_heads < 1 || L.heads % L.kv_heads || L.dim < 1 || L.dim_pad < L.dim || (L.dim_pad & 63) || L.dim_pad > 256 ||
          L.vdim_pad < 64 || (L.vdim_pad & 63) || L.vdim_pad > 256 || L.q_temp_every < 1)
        return fail(LCC_ERR_SHAPE, "decoder layer %d: attention sizes", (int)i);
      o.kv = off; off += align_up(Lmax * L.kv_heads * L.dim_pad, 128);
      o.v = off; off += align_up(Lmax * L.kv_heads * L.vdim_pad, 128);
    }
    o.state = off; off += align_up((size_t)2 * L.rec_heads * L.rec_key_pad * L.rec_vdim_pad, 128);
    if (L.rec_conv_taps) { o.conv = off; off += align_up((size_t)2 * L.rec_conv_taps * conv_channels(L), 128); }
  }
  e->dec_kv_total = off;
  return 0;
}
int mixers_resolve_weights(lcc_engine* e, std::string* missing) {
  auto get = [&](const std::string& n) -> const bf16_t* {
    auto it = e->w.find(n);
    if (it == e->w.end()) { if (missing) { *missing += n; *missing += ' '; } return nullptr; }
    return (const bf16_t*)it->second;
  };
  e->embed = get("embed"); e->dec_bigram = get("bigram"); e->lm_head = get("lm_head"); e->dec_final_w = get("final_norm");
  for (size_t i = 0; i < e->dl.size(); ++i) {
    const lcc_decoder_layer& L = e->dl[i];
    const std::string p = "dec." + std::to_string(i) + ".";
    DecLayerW& w = e->dw[i];
    w.norm1 = get(p + "norm1"); w.norm1b = get(p + "norm1b"); w.in_w = get(p + "in_w"); w.rec_norm = get(p + "rec_norm"); w.ro_w = get(p + "ro_w");
    w.rec_rate = (const float*)get(p + "rec_rate");
    if (has_attn(L)) {
      w.q_norm = get(p + "q_norm"); w.k_norm = get(p + "k_norm"); w.slope = (const float*)get(p + "slope"); w.lo_w = get(p + "lo_w");
      w.l_out = get(p + "l_out"); w.r_out = get(p + "r_out");
    } else {
      w.conv_w = get(p + "conv_w"); w.conv_b = get(p + "conv_b"); w.rec_dt_bias = (const float*)get(p + "rec_dt_bias"); w.rec_skip = (const float*)get(p + "rec_skip");
    }
    if (L.ff_pad > 0) { w.norm2 = get(p + "norm2"); w.norm2b = get(p + "norm2b"); w.gate_up_w = get(p + "gate_up_w"); w.down_w = get(p + "down_w"); }
  }
  return missing && !missing->empty() ? LCC_ERR_STATE : 0;
}

// S packed rows through every layer; pt null: a decode step over the streams `d_slots`.  On exit b.h holds the final norm of the residual.
int run_mixer_layers(lcc_engine* e, const DecBuffers& b, int S, const PrefillTables* pt, const int32_t* d_slots, int nsplit_attn, const AttnDirect& direct, hipStream_t st) {
  const bool fused = !pt && S <= 16 && g_fused_decode;
  const int W = e->c.hidden_size, NL = (int)e->dl.size();
  if (e->llm_over) return fail(LCC_ERR_STATE, "per-layer input overrides are not available for this model family");
  auto product = [&](const bf16_t* X, int ldx, const bf16_t* w, int N, int K, float* out, size_t cap, int* ns) {       // fp32 slabs of X W^T
    if (!fused) return slab_gemm(b, X, ldx, w, S, N, K, ns, st, out, cap);
    DgArgs g; g.W = w; g.M = S; g.N = N; g.K = K; g.X = X; g.ldx = ldx; g.C32 = out; g.ldc = N;
    *ns = 1;
    return dgemv_f32(g, st);
  };
  LCC_TRY(tap(e, b, 0, S, st));
  for (int l = 0; l < NL; ++l) {
    const lcc_decoder_layer& L = e->dl[l];
    const DecLayerW& w = e->dw[l];
    const DecOffsets& off = e->dec_off[l];
    const int in_n = in_rows(L), rin = rec_inner(L);
    const bf16_t* after = l + 1 < NL ? e->dw[l + 1].norm1 : e->dec_final_w;      // the norm behind this layer
    int ns = 1;
    LCC_TRY(product(b.h, W, w.in_w, in_n, W, b.part, b.part_cap, &ns));

    GqaInArgs gi;
    if (has_attn(L)) {
      gi.part = b.part; gi.nsplit = ns; gi.rows = S; gi.ldn = in_n; gi.heads = L.heads; gi.kv_heads = L.kv_heads; gi.dim = L.dim; gi.dim_pad = L.dim_pad;
      gi.vdim_pad = L.vdim_pad; gi.eps = e->dc.norm_eps; gi.q_norm = w.q_norm; gi.k_norm = w.k_norm; gi.temp_coef = L.q_temp_coef; gi.temp_every = L.q_temp_every;
      gi.q = b.q; gi.tok_stream = pt ? pt->tok_stream : d_slots; gi.tok_pos = pt ? pt->tok_pos : nullptr; gi.kv_len = e->d_kv_len; gi.kv_base = e->d_kv_base;
      gi.k_off = off.kv; gi.v_off = off.v; gi.lmax = e->lim.max_kv_len;
    }
    RecInArgs ri = rec_cols(L);
    ri.part = b.part; ri.nsplit = ns; ri.rows = S; ri.conv_w = w.conv_w; ri.conv_b = w.conv_b; ri.rate = w.rec_rate; ri.dt_bias = w.rec_dt_bias; ri.skip = w.rec_skip;
    ri.tok_stream = gi.tok_stream = pt ? pt->tok_stream : d_slots; ri.kv_base = e->d_kv_base; ri.state_off = off.state; ri.conv_off = off.conv;
    if (pt) { ri.tok_pos = pt->tok_pos; ri.tok_row0 = pt->tok_row0; ri.tok_last = pt->tok_last; }
    ri.kv_len = e->d_kv_len; ri.done = e->d_done; ri.q = b.rq; ri.k = b.rk; ri.v = b.rv; ri.dt = b.dt;
    RecNormArgs rn; rn.y = b.y; rn.part = b.part; rn.nsplit = ns; rn.rows = S; rn.ldn = in_n; rn.gate_col = gate_col(L); rn.gate_first = L.mixer == LCC_MIXER_SSD;
    rn.heads = L.rec_heads; rn.vdim = L.rec_vdim; rn.ep = L.rec_vdim_pad; rn.norm_groups = L.rec_norm_groups; rn.eps = e->dc.norm_eps; rn.w = w.rec_norm;
    rn.out = b.rec; rn.ld = rin;
    const float scale_log2e = L.scale * 1.4426950408889634f;
    if (pt) {
      LCC_TRY(mixer_prep(has_attn(L) ? &gi : nullptr, &ri, st));
      if (has_attn(L)) {
        MhaArgs a; a.q = b.q; a.out = b.att; a.ldo = L.heads * L.vdim_pad; a.grp_q0 = pt->grp_q0; a.grp_nq = pt->grp_nq; a.grp_pos0 = pt->grp_pos0;
        a.grp_slot = pt->grp_slot; a.n_groups = pt->n_grps; a.rows = S; a.heads = L.heads; a.dim = L.dim_pad; a.vdim = L.vdim_pad; a.scale_log2e = scale_log2e;
        a.kv_base = e->d_kv_base; a.k_off = off.kv; a.v_off = off.v; a.lmax = e->lim.max_kv_len; a.kv_heads = L.kv_heads; a.slope = w.slope;
        LCC_TRY(attn_mha(a, st));
      }
      RecScanArgs s; s.q = b.rq; s.k = b.rk; s.v = b.rv; s.dt = ri.dt_col >= 0 ? b.dt : nullptr; s.rate = w.rec_rate; s.skip = w.rec_skip; s.y = b.y;
      s.heads = L.rec_heads; s.groups = L.rec_groups; s.np = L.rec_key_pad; s.ep = L.rec_vdim_pad; s.seg_row0 = pt->seg_row0; s.seg_rows = pt->seg_rows;
      s.seg_slot = pt->seg_slot; s.seg_fresh = pt->seg_fresh; s.n_seg = pt->n_seg; s.str_seg0 = pt->str_seg0; s.str_nseg = pt->str_nseg; s.n_streams = pt->n_streams;
      if (s.n_seg > s.n_streams && s.n_seg > b.seg_cap) return fail(LCC_ERR_STATE, "%d segments, workspace for %d", s.n_seg, b.seg_cap);
      s.seg_state = b.seg_state; s.seg_decay = b.seg_decay; s.kv_base = e->d_kv_base; s.state_off = off.state;
      LCC_TRY(rec_scan(s, st));
      if (ri.taps) rn.conv = &ri;
      LCC_TRY(rec_norm(rn, st));
    } else {
      ri.direct = gi.direct = direct;
      if (has_attn(L)) {
        GqaDecodeArgs a; a.q = b.q; a.rows = S; a.heads = L.heads; a.kv_heads = L.kv_heads; a.dim = L.dim_pad; a.vdim = L.vdim_pad; a.nsplit = nsplit_attn;
        a.scale_log2e = scale_log2e; a.slope = w.slope; a.slots = d_slots; a.kv_len = e->d_kv_len; a.kv_base = e->d_kv_base; a.k_off = off.kv; a.v_off = off.v;
        a.lmax = e->lim.max_kv_len; a.ws_o = b.ws_o; a.ws_ml = b.ws_ml; a.out = b.att; a.direct = direct;
        if (fused && rec_gqa_decode_ok(ri, a)) {
          LCC_TRY(rec_gqa_decode(ri, gi, a, b.y, st));
        } else {
          LCC_TRY(rec_decode(ri, &gi, b.y, st));
          LCC_TRY(gqa_decode(a, st));
        }
        LCC_TRY(gqa_merge_rec_norm(a, rn, st));
      } else {
        LCC_TRY(rec_decode(ri, nullptr, b.y, st));
        LCC_TRY(rec_norm(rn, st));
      }
    }

    // output product(s), the norms around the residual
    PostNormArgs pn; pn.part = b.part; pn.post_w = w.norm1b; pn.next_w = L.ff_pad > 0 ? w.norm2 : after; pn.x = b.x; pn.h = b.h; pn.rows = S; pn.width = e->dc.width;
    pn.dim = W; pn.eps = e->dc.norm_eps;
    if (has_attn(L)) {
      const int kl = L.heads * L.vdim_pad;
      const size_t half = b.part_cap / 2 / 64 * 64;
      float* part_b = b.part + half;
      pn.part_b = part_b; pn.w_a = w.l_out; pn.w_b = w.r_out;
      if (fused) {
        DgArgs ga, gb;
        ga.W = w.lo_w; ga.M = S; ga.N = W; ga.K = kl; ga.X = b.att; ga.ldx = kl; ga.C32 = b.part; ga.ldc = W;
        gb.W = w.ro_w; gb.M = S; gb.N = W; gb.K = rin; gb.X = b.rec; gb.ldx = rin; gb.C32 = part_b; gb.ldc = W;
        LCC_TRY(dgemv_f32_pair(ga, gb, st));
      } else {
        LCC_TRY(slab_gemm(b, b.att, kl, w.lo_w, S, W, kl, &pn.nsplit, st, b.part, half));
        LCC_TRY(slab_gemm(b, b.rec, rin, w.ro_w, S, W, rin, &pn.nsplit_b, st, part_b, half));
      }
    } else {
      LCC_TRY(product(b.rec, rin, w.ro_w, W, rin, b.part, b.part_cap, &pn.nsplit));
    }
    LCC_TRY(post_norm_resid(pn, st));

    if (L.ff_pad > 0) {
      if (fused) {
        DgArgs g; g.W = w.gate_up_w; g.M = S; g.N = 2 * L.ff_pad; g.K = W; g.X = b.h; g.ldx = W; g.C = b.act; g.ldc = L.ff_pad;
        LCC_TRY(dgemv_swiglu(g, st));
      } else {
        LCC_TRY(plain_gemm(b.h, W, w.gate_up_w, b.act, L.ff_pad, S, 2 * L.ff_pad, W, LCC_EPI_SWIGLU, st));
      }
      PostNormArgs pf; pf.part = b.part; pf.post_w = w.norm2b; pf.next_w = after; pf.x = b.x; pf.h = b.h; pf.rows = S; pf.width = e->dc.width; pf.dim = W;
      pf.eps = e->dc.norm_eps;
      LCC_TRY(product(b.act, L.ff_pad, w.down_w, W, L.ff_pad, b.part, b.part_cap, &pf.nsplit));
      LCC_TRY(post_norm_resid(pf, st));
    }
    LCC_TRY(tap(e, b, l + 1, S, st));
  }
  return 0;
}
