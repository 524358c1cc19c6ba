// Row operators of the layer-list decoders (engine_decoder.hip): embedding, residual add and norm, logits.
//
// The residual stream is fp32 from the embedding to the last norm.  Two block forms: one norm in front of parallel sublayers (Dynamic Tanh), or a
// norm before and after every sublayer (RMS norms, weights stored around zero; further down).  Dynamic Tanh, y = tanh(alpha x) w + b: it needs no row
// statistic, so it runs in the pass that writes the residual -- the consumer GEMM reads ready bf16 activations and no launch exists for the
// norm alone.  Rows are padded to a multiple of 64 channels with zero weights, so a padding channel stays 0 through the norm (w = b = 0).
#include "common.h"
#include "kernels.h"
#include "latent_ops.h"

namespace lcc {

LCC_DEVICE u32x4 dyt8(const float (&x)[8], float alpha, const bf16_t* w, const bf16_t* b) {
  const u32x4 wv = ld16(w), bv = ld16(b);
  u32x4 o;
#pragma unroll
  for (int e = 0; e < 4; ++e)
    o[e] = pack2(dyt_value(x[2 * e], alpha, lo2f(wv[e]), lo2f(bv[e])), dyt_value(x[2 * e + 1], alpha, hi2f(wv[e]), hi2f(bv[e])));
  return o;
}

// x = embedding row (fp32), h = norm(x).  ids[i], or -- decode -- the slot's current token ids[indirect[i]].
__global__ __launch_bounds__(256) void embed_dyt_kernel(const int32_t* __restrict__ ids, const int32_t* __restrict__ indirect,
                                                        const bf16_t* __restrict__ table, DytNorm nm, float* __restrict__ x,
                                                        bf16_t* __restrict__ h, int rows, int dim) {
  const int cpr = dim >> 3;
  const float alpha = bf2f(nm.alpha[0]);
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < (int64_t)rows * cpr; i += (int64_t)gridDim.x * 256) {
    const int r = (int)(i / cpr), c = (int)(i - (int64_t)r * cpr) * 8;
    const int id = indirect ? ids[indirect[r]] : ids[r];
    const u32x4 q = ld16(table + (size_t)id * dim + c);
    float v[8];
#pragma unroll
    for (int e = 0; e < 4; ++e) { v[2 * e] = lo2f(q[e]); v[2 * e + 1] = hi2f(q[e]); }
    float* xp = x + (size_t)r * dim + c;
    *reinterpret_cast<f32x4*>(xp) = (f32x4){v[0], v[1], v[2], v[3]};
    *reinterpret_cast<f32x4*>(xp + 4) = (f32x4){v[4], v[5], v[6], v[7]};
    st16(h + (size_t)r * dim + c, dyt8(v, alpha, nm.w + c, nm.b + c));
  }
}

// x += sum of the nsplit fp32 slabs of the layer's output product, h = norm(x) of the NEXT norm
__global__ __launch_bounds__(256) void resid_dyt_kernel(float* __restrict__ x, const float* __restrict__ part, int nsplit, DytNorm nm,
                                                        bf16_t* __restrict__ h, int rows, int dim) {
  const int cpr = dim >> 3;
  const float alpha = bf2f(nm.alpha[0]);
  const size_t slab = (size_t)rows * dim;
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < (int64_t)rows * cpr; i += (int64_t)gridDim.x * 256) {
    const int c = (int)(i % cpr) * 8;
    const size_t off = (size_t)i * 8;
    f32x4 a = *reinterpret_cast<const f32x4*>(x + off), b = *reinterpret_cast<const f32x4*>(x + off + 4);
    f32x4 sa = {0.f, 0.f, 0.f, 0.f}, sb = {0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < nsplit; ++s) {
      sa += *reinterpret_cast<const f32x4*>(part + s * slab + off);
      sb += *reinterpret_cast<const f32x4*>(part + s * slab + off + 4);
    }
    a += sa; b += sb;
    *reinterpret_cast<f32x4*>(x + off) = a;
    *reinterpret_cast<f32x4*>(x + off + 4) = b;
    const float v[8] = {a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
    st16(h + off, dyt8(v, alpha, nm.w + c, nm.b + c));
  }
}

// logits = cap * tanh(z / cap) (cap <= 0: z) of z = scale * the sum of the fp32 slabs [nsplit][rows][ld]; ids past the vocabulary are -inf.  `out` [rows][ld]
// feeds the sampler, `dense` [rows][vocab] (optional) is the caller's copy.
__global__ __launch_bounds__(256) void logits_cap_kernel(const float* __restrict__ part, int nsplit, int rows, int ld, int vocab, float scale,
                                                         float cap, float* __restrict__ out, float* __restrict__ dense) {
  const size_t slab = (size_t)rows * ld;
  const float inv = cap > 0.f ? 1.f / cap : 0.f;
  for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < slab; i += (size_t)gridDim.x * 256) {
    const int r = (int)(i / ld), n = (int)(i - (size_t)r * ld);
    float z = 0.f;
    for (int s = 0; s < nsplit; ++s) z += part[s * slab + i];
    z *= scale;
    if (cap > 0.f) z = cap * tanhf(z * inv);
    if (out) out[i] = n < vocab ? z : -INFINITY;
    if (dense && n < vocab) dense[(size_t)r * vocab + n] = z;
  }
}

// ---- RMS norms with weights stored around zero: one block of NW waves per row, two 4-channel pieces per thread ----
LCC_DEVICE f32x4 bf4(u32x2 q) { return (f32x4){lo2f(q.x), hi2f(q.x), lo2f(q.y), hi2f(q.y)}; }
LCC_DEVICE float sq4(f32x4 v) { return (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]); }
// sum of the slabs, four of them in flight
LCC_DEVICE f32x4 slabs4(const float* part, int nsplit, size_t slab, size_t at) {
  f32x4 v = *reinterpret_cast<const f32x4*>(part + at);
  for (int k = 1; k < nsplit; k += 4) {
    f32x4 u[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) u[j] = *reinterpret_cast<const f32x4*>(part + (size_t)min(k + j, nsplit - 1) * slab + at);
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (k + j < nsplit) v += u[j];
  }
  return v;
}
LCC_DEVICE float inv_rms(float sum, int n, float eps) { return 1.f / sqrtf(sum / (float)n + eps); }

template <int NW>
__global__ __launch_bounds__(NW * 64) void embed_bigram_rms_kernel(const int32_t* __restrict__ ids, const int32_t* __restrict__ tok_stream,
                                                               const int32_t* __restrict__ tok_pos, const int32_t* __restrict__ tok_row0,
                                                               const int32_t* __restrict__ kv_len, const int32_t* __restrict__ prev_tok,
                                                               const bf16_t* __restrict__ table, BigramEmbed bg, const bf16_t* __restrict__ norm_w, float eps,
                                                               float* __restrict__ x, bf16_t* __restrict__ h, int width, int dim) {
  constexpr int MAXC = 2;
  __shared__ float red[NW];
  const int row = blockIdx.x, tid = threadIdx.x, slot = tok_stream[row];
  const int id = tok_pos ? ids[row] : ids[slot], pos = tok_pos ? tok_pos[row] : kv_len[slot];
  const int prev = tok_pos && tok_row0[row] != row ? ids[row - 1] : prev_tok[slot];
  const int64_t bucket = pos == 0 ? bg.buckets : ((int64_t)prev * bg.mul_prev + (int64_t)id * bg.mul_cur) % bg.buckets;
  const bf16_t *e = table + (size_t)id * dim, *b = bg.table + (size_t)bucket * dim;
  f32x4 v[MAXC];
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < MAXC; ++i) {
    const int c = (tid + NW * 64 * i) * 4;
    if (c < dim) {
      v[i] = bf4(ld8(e + c)) + bf4(ld8(b + c));
      *reinterpret_cast<f32x4*>(x + (size_t)row * dim + c) = v[i];
      s += sq4(v[i]);
    }
  }
  const float r = inv_rms(block_sum<NW>(s, red), width, eps);
#pragma unroll
  for (int i = 0; i < MAXC; ++i) {
    const int c = (tid + NW * 64 * i) * 4;
    if (c < dim) {
      const f32x4 y = v[i] * r * (1.f + bf4(ld8(norm_w + c)));
      st8(h + (size_t)row * dim + c, (u32x2){pack2(y[0], y[1]), pack2(y[2], y[3])});
    }
  }
}

template <int NW, bool PAIR>
__global__ __launch_bounds__(NW * 64) void post_norm_resid_kernel(PostNormArgs a) {
  constexpr int MAXC = 2;
  __shared__ float red[NW], red2[NW];
  const int row = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const size_t slab = (size_t)a.rows * a.dim, at = (size_t)row * a.dim;
  f32x4 y[MAXC], yb[PAIR ? MAXC : 1], xv[MAXC];
  u32x2 wp[MAXC], wn[MAXC], wa[PAIR ? MAXC : 1], wb[PAIR ? MAXC : 1];
  float s = 0.f, sb = 0.f;
#pragma unroll
  for (int i = 0; i < MAXC; ++i) {
    const int c = (tid + NW * 64 * i) * 4, j = PAIR ? i : 0;
    y[i] = xv[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
    wp[i] = wn[i] = (u32x2){0u, 0u};
    if (PAIR) { yb[j] = y[i]; wa[j] = wb[j] = wp[i]; }
    if (c < a.dim) {
      xv[i] = *reinterpret_cast<const f32x4*>(a.x + at + c);
      wp[i] = ld8(a.post_w + c); wn[i] = ld8(a.next_w + c);
      y[i] = slabs4(a.part, a.nsplit, slab, at + c);
      s += sq4(y[i]);
      if (PAIR) {
        wa[j] = ld8(a.w_a + c); wb[j] = ld8(a.w_b + c);
        yb[j] = slabs4(a.part_b, a.nsplit_b, slab, at + c);
        sb += sq4(yb[j]);
      }
    }
  }
  if (PAIR) {
    s = wave_sum(s); sb = wave_sum(sb);
    if (lane == 0) { red[wave] = s; red2[wave] = sb; }
    __syncthreads();
    s = sb = 0.f;
#pragma unroll
    for (int k = 0; k < NW; ++k) { s += red[k]; sb += red2[k]; }
    const float ra = 0.5f * inv_rms(s, a.width, a.eps), rb = 0.5f * inv_rms(sb, a.width, a.eps);
    s = 0.f;
#pragma unroll
    for (int i = 0; i < MAXC; ++i) {
      const int j = PAIR ? i : 0;
      y[i] = y[i] * ra * bf4(wa[j]) + yb[j] * rb * bf4(wb[j]);
      s += sq4(y[i]);
    }
  }
  const float r = inv_rms(block_sum<NW>(s, red), a.width, a.eps);
  s = 0.f;
#pragma unroll
  for (int i = 0; i < MAXC; ++i) {
    xv[i] += y[i] * r * (1.f + bf4(wp[i]));
    s += sq4(xv[i]);
  }
  const float rn = inv_rms(block_sum<NW>(s, red2), a.width, a.eps);
#pragma unroll
  for (int i = 0; i < MAXC; ++i) {
    const int c = (tid + NW * 64 * i) * 4;
    if (c < a.dim) {
      *reinterpret_cast<f32x4*>(a.x + at + c) = xv[i];
      const f32x4 o = xv[i] * rn * (1.f + bf4(wn[i]));
      st8(a.h + at + c, (u32x2){pack2(o[0], o[1]), pack2(o[2], o[3])});
    }
  }
}

// the caller's own continuation: the token a slot consumes in its next decode step; its generate counters restart as after a prefill
__global__ void set_tokens_kernel(const int32_t* __restrict__ slots, const int32_t* __restrict__ toks, int n, int32_t* __restrict__ cur_tok,
                                  int32_t* __restrict__ done, int32_t* __restrict__ hist_col) {
  const int i = blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= n) return;
  const int s = slots[i];
  cur_tok[s] = toks[i]; done[s] = 0; hist_col[s] = 0;
}

static unsigned grid_for(int64_t items) { return (unsigned)((items + 255) / 256 < 4096 ? (items + 255) / 256 : 4096); }

static bool dyt_ok(const DytNorm& n) { return n.w && n.b && n.alpha && ((((uintptr_t)n.w) | ((uintptr_t)n.b)) & 15) == 0; }
int embed_dyt(const int32_t* ids, const int32_t* indirect, const bf16_t* table, const DytNorm& nm, float* x, bf16_t* h, int rows, int dim, hipStream_t st) {
  if (rows <= 0) return 0;
  if (dim <= 0 || (dim & 7)) return LCC_ERR_SHAPE;
  if (!ids || !table || !x || !h || !dyt_ok(nm)) return LCC_ERR_ARG;
  embed_dyt_kernel<<<dim3(grid_for((int64_t)rows * (dim >> 3))), dim3(256), 0, st>>>(ids, indirect, table, nm, x, h, rows, dim);
  return 0;
}
int resid_dyt(float* x, const float* part, int nsplit, const DytNorm& nm, bf16_t* h, int rows, int dim, hipStream_t st) {
  if (rows <= 0) return 0;
  if (dim <= 0 || (dim & 7) || nsplit < 0) return LCC_ERR_SHAPE;
  if (!x || !h || (nsplit > 0 && !part) || !dyt_ok(nm)) return LCC_ERR_ARG;
  resid_dyt_kernel<<<dim3(grid_for((int64_t)rows * (dim >> 3))), dim3(256), 0, st>>>(x, part, nsplit, nm, h, rows, dim);
  return 0;
}
int logits_cap(const float* part, int nsplit, int rows, int ld, int vocab, float scale, float cap, float* out, float* dense, hipStream_t st) {
  if (rows <= 0) return 0;
  if (nsplit < 1 || vocab < 1 || ld < vocab) return LCC_ERR_SHAPE;
  if (!part || (!out && !dense)) return LCC_ERR_ARG;
  logits_cap_kernel<<<dim3(grid_for((int64_t)rows * ld)), dim3(256), 0, st>>>(part, nsplit, rows, ld, vocab, scale, cap, out, dense);
  return 0;
}
int embed_bigram_rms(const int32_t* ids, const int32_t* tok_stream, const int32_t* tok_pos, const int32_t* tok_row0, const int32_t* kv_len, const int32_t* prev_tok,
                     const bf16_t* table, const BigramEmbed& bg, const bf16_t* norm_w, float eps, float* x, bf16_t* h, int rows, int width, int dim, hipStream_t st) {
  if (rows <= 0) return 0;
  if (dim <= 0 || (dim & 7) || dim > 8192 || width < 1 || width > dim || bg.buckets < 1) return LCC_ERR_SHAPE;
  if (!ids || !tok_stream || (tok_pos ? !tok_row0 : !kv_len) || !prev_tok || !table || !bg.table || !norm_w || !x || !h) return LCC_ERR_ARG;
#define LCC_GO(C) embed_bigram_rms_kernel<C><<<dim3(rows), dim3(C * 64), 0, st>>>(ids, tok_stream, tok_pos, tok_row0, kv_len, prev_tok, table, bg, norm_w, eps, x, h, width, dim)
  if (dim <= 2048) LCC_GO(4); else if (dim <= 4096) LCC_GO(8); else LCC_GO(16);
#undef LCC_GO
  return 0;
}
int post_norm_resid(const PostNormArgs& a, hipStream_t st) {
  if (a.rows <= 0) return 0;
  if (a.dim <= 0 || (a.dim & 7) || a.dim > 8192 || a.width < 1 || a.width > a.dim || a.nsplit < 1 || (a.part_b && a.nsplit_b < 1)) return LCC_ERR_SHAPE;
  if (!a.part || !a.post_w || !a.next_w || !a.x || !a.h || (a.part_b && (!a.w_a || !a.w_b))) return LCC_ERR_ARG;
#define LCC_GO(C)                                                                                 \
  do {                                                                                            \
    if (a.part_b) post_norm_resid_kernel<C, true><<<dim3(a.rows), dim3(C * 64), 0, st>>>(a);      \
    else post_norm_resid_kernel<C, false><<<dim3(a.rows), dim3(C * 64), 0, st>>>(a);              \
  } while (0)
  if (a.dim <= 2048) LCC_GO(4); else if (a.dim <= 4096) LCC_GO(8); else LCC_GO(16);
#undef LCC_GO
  return 0;
}
int set_tokens(const int32_t* slots, const int32_t* toks, int n, int32_t* cur_tok, int32_t* done, int32_t* hist_col, hipStream_t st) {
  if (n <= 0) return 0;
  set_tokens_kernel<<<dim3((n + 63) / 64), dim3(64), 0, st>>>(slots, toks, n, cur_tok, done, hist_col);
  return 0;
}

}  // namespace lcc
