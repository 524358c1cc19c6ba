// Device code shared by recurrent.hip and biased_attn.hip: a new row behind the fused input projection of a mixer, and small fp32 helpers.
#pragma once
#include "common.h"
#include "kernels.h"

namespace lcc {

typedef __attribute__((ext_vector_type(4))) short tr16x4;
// ds_read_b64_tr_b16: in a group of 16 lanes, lane l supplies 4 consecutive channels of row l / 4 and receives channel l of the 4 rows
LCC_DEVICE u32x2 lds_read_tr(const void* p) {
  return __builtin_bit_cast(u32x2, __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) tr16x4*)(p)));
}
LCC_DEVICE f32x4 unpack4(u32x2 q) { return (f32x4){lo2f(q.x), hi2f(q.x), lo2f(q.y), hi2f(q.y)}; }
LCC_DEVICE u32x2 pack4(f32x4 v) { return (u32x2){pack2(v[0], v[1]), pack2(v[2], v[3])}; }
LCC_DEVICE float sigmoid_f(float z) { return 1.f / (1.f + __expf(-z)); }
LCC_DEVICE float silu_f(float z) { return z / (1.f + __expf(-z)); }
LCC_DEVICE float softplus_f(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
LCC_DEVICE f32x4 silu4(f32x4 z) { return (f32x4){silu_f(z[0]), silu_f(z[1]), silu_f(z[2]), silu_f(z[3])}; }
LCC_DEVICE f32x4 slab_sum4(const float* part, int nsplit, size_t slab, size_t off) {
  f32x4 v = *reinterpret_cast<const f32x4*>(part + off);
  for (int s = 1; s < nsplit; ++s) v += *reinterpret_cast<const f32x4*>(part + s * slab + off);
  return v;
}

// Queries (normed, scaled by the position's temperature) to a.q, keys (normed) and values to the slot's cache.  All threads of a block of NW waves.
template <int NW>
LCC_DEVICE void gqa_row(const GqaInArgs& a, int row) {
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const size_t slab = (size_t)a.rows * a.ldn, at = (size_t)row * a.ldn;
  int pos;
  bf16_t* arena;
  if (a.direct.used) { pos = a.direct.n[row & 3] - 1; arena = const_cast<bf16_t*>(a.direct.base[row & 3]); }
  else { const int slot = a.tok_stream[row]; pos = a.tok_pos ? a.tok_pos[row] : a.kv_len[slot]; arena = a.kv_base[slot]; }
  const float temp = 1.f + a.temp_coef * logf((float)((pos + 1) / a.temp_every) + 1.f);
  for (int h = wave; h < a.heads + a.kv_heads; h += NW) {
    const bool isq = h < a.heads;
    const int c = lane * 4;                            // dim_pad <= 256
    f32x4 v = {0.f, 0.f, 0.f, 0.f}, w = v;
    if (c < a.dim_pad) {
      v = slab_sum4(a.part, a.nsplit, slab, at + (size_t)h * a.dim_pad + c);
      w = unpack4(ld8((isq ? a.q_norm : a.k_norm) + c));
    }
    const float ss = wave_sum((v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]));
    const float r = (isq ? temp : 1.f) / sqrtf(ss / (float)a.dim + a.eps);
    if (c < a.dim_pad) {
      bf16_t* dst = isq ? a.q + ((size_t)row * a.heads + h) * a.dim_pad : arena + a.k_off + ((size_t)(h - a.heads) * a.lmax + pos) * a.dim_pad;
      st8(dst + c, pack4(v * r * w));
    }
  }
  const int vcol = (a.heads + a.kv_heads) * a.dim_pad, nv = a.kv_heads * a.vdim_pad;
  for (int c = tid * 4; c < nv; c += NW * 256) {
    const f32x4 v = slab_sum4(a.part, a.nsplit, slab, at + vcol + c);
    const int g = c / a.vdim_pad, d = c - g * a.vdim_pad;
    bf16_t* dst = arena + a.v_off + (size_t)g * a.lmax * a.vdim_pad + ((size_t)(pos >> 5) * a.vdim_pad + d) * 32 + (pos & 31);
#pragma unroll
    for (int e = 0; e < 4; ++e) dst[e * 32] = f2bf(v[e]);
  }
}

// Four channels of a recurrent mixer's activated input at `col` of the projection: silu of the value, or of the short causal convolution over the
// projection's rows (rows of this call from r0 on, older ones out of the slot's ring: position p at row p % taps, zeros before the start).
LCC_DEVICE f32x4 rec_in4(const RecInArgs& a, int row, int r0, int pos, const float* ring, int col, f32x4* raw) {
  const size_t slab = (size_t)a.rows * a.ldn;
  const f32x4 u = slab_sum4(a.part, a.nsplit, slab, (size_t)row * a.ldn + col);
  *raw = u;
  if (a.taps == 0) return silu4(u);
  const int ch = col - a.conv_col;
  f32x4 acc = unpack4(ld8(a.conv_b + ch)) + unpack4(ld8(a.conv_w + (size_t)(a.taps - 1) * a.conv_ch + ch)) * u;
  for (int back = 1; back < a.taps && back <= pos; ++back) {
    const f32x4 p = row - back >= r0 ? slab_sum4(a.part, a.nsplit, slab, (size_t)(row - back) * a.ldn + col)
                                     : *reinterpret_cast<const f32x4*>(ring + (size_t)((pos - back) % a.taps) * a.conv_ch + ch);
    acc += unpack4(ld8(a.conv_w + (size_t)(a.taps - 1 - back) * a.conv_ch + ch)) * p;
  }
  return silu4(acc);
}
LCC_DEVICE float rec_dt(const RecInArgs& a, int row, int h) {
  if (a.dt_col < 0) return 1.f;
  const float* p = a.part + (size_t)row * a.ldn + a.dt_col + h;
  float z = p[0];
  for (int s = 1; s < a.nsplit; ++s) z += p[(size_t)s * a.rows * a.ldn];
  return softplus_f(z + a.dt_bias[h]);
}
// one (row, norm group) of the gated norm behind the recurrence, by a block of NW waves; red: NW floats of LDS.  Up to MAXP pieces of 4 channels per
// thread stay in registers between the statistic and the result.
template <int NW, int MAXP>
LCC_DEVICE void rec_norm_row(const RecNormArgs& a, int row, int grp, float* red) {
  const int tid = threadIdx.x, inner = a.heads * a.vdim, gs = inner / a.norm_groups, nt = NW * 64;
  const size_t slab = (size_t)a.rows * a.ldn;
  const float* y = a.y + (size_t)row * a.heads * a.ep;
  const size_t gate = (size_t)row * a.ldn + a.gate_col;
  bf16_t* out = a.out + (size_t)row * a.ld;
  const int lo = grp * gs, hi = lo + gs;
  float ss = 0.f;
  if (((a.vdim | gs) & 3) == 0 && gs <= nt * 4 * MAXP) {      // pieces of 4 channels stay inside a head and a group
    f32x4 v[MAXP], g[MAXP];
    u32x2 w[MAXP];
#pragma unroll
    for (int i = 0; i < MAXP; ++i) {
      const int r = lo + (tid + i * nt) * 4;
      v[i] = g[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
      w[i] = (u32x2){0u, 0u};
      if (r < hi) {
        const int h = r / a.vdim, c = h * a.ep + r - h * a.vdim;
        v[i] = *reinterpret_cast<const f32x4*>(y + c);
        g[i] = slab_sum4(a.part, a.nsplit, slab, gate + c);
        w[i] = ld8(a.w + r);
      }
    }
#pragma unroll
    for (int i = 0; i < MAXP; ++i) {
      if (a.gate_first) v[i] *= silu4(g[i]);
      ss += (v[i][0] * v[i][0] + v[i][1] * v[i][1]) + (v[i][2] * v[i][2] + v[i][3] * v[i][3]);
    }
    const float inv = 1.f / sqrtf(block_sum<NW>(ss, red) / (float)gs + a.eps);
#pragma unroll
    for (int i = 0; i < MAXP; ++i) {
      const int r = lo + (tid + i * nt) * 4;
      if (r < hi) {
        f32x4 o = v[i] * inv * unpack4(w[i]);
        if (!a.gate_first) o *= (f32x4){sigmoid_f(g[i][0]), sigmoid_f(g[i][1]), sigmoid_f(g[i][2]), sigmoid_f(g[i][3])};
        st8(out + r, pack4(o));
      }
    }
  } else {
    auto gate1 = [&](int c) {
      float z = a.part[gate + c];
      for (int s = 1; s < a.nsplit; ++s) z += a.part[s * slab + gate + c];
      return z;
    };
    for (int r = lo + tid; r < hi; r += nt) {
      const int h = r / a.vdim, c = h * a.ep + r - h * a.vdim;
      const float v = a.gate_first ? y[c] * silu_f(gate1(c)) : y[c];
      ss += v * v;
    }
    const float inv = 1.f / sqrtf(block_sum<NW>(ss, red) / (float)gs + a.eps);
    for (int r = lo + tid; r < hi; r += nt) {
      const int h = r / a.vdim, c = h * a.ep + r - h * a.vdim;
      const float g = gate1(c), f = inv * bf2f(a.w[r]);
      out[r] = f2bf(a.gate_first ? y[c] * silu_f(g) * f : y[c] * f * sigmoid_f(g));
    }
  }
  if (grp == 0)
    for (int r = inner + tid; r < a.ld; r += nt) out[r] = 0;
}
// the last inputs of a stream's portion, for the convolution of its next call
template <int NW>
LCC_DEVICE void conv_ring_row(const RecInArgs& a, int row) {
  if (a.tok_last[row] - row >= a.taps) return;
  float* ring = reinterpret_cast<float*>(a.kv_base[a.tok_stream[row]] + a.conv_off) + (size_t)(a.tok_pos[row] % a.taps) * a.conv_ch;
  for (int c = threadIdx.x * 4; c < a.conv_ch; c += NW * 256)
    *reinterpret_cast<f32x4*>(ring + c) = slab_sum4(a.part, a.nsplit, (size_t)a.rows * a.ldn, (size_t)row * a.ldn + a.conv_col + c);
}

// One wave of the decode attention: a key split of one row, KV head and tile of 16 query heads of it; partial (O, m, l) to the workspace.  A 32-key tile
// is two 16-key MFMA row tiles whose rows are dealt so that the probabilities a lane ends up with are the 8 consecutive keys its operand of
// the P.V product needs.  NEW: queries, the new key and the new value come straight from the input projection (one slab), the last split
// puts the new token into its operands and the cache.
template <int DK, int DV, bool NEW>
LCC_DEVICE void gqa_decode_wave(const GqaDecodeArgs& a, const GqaInArgs& in, int split, int kvh, int tile, int b) {
  constexpr int KS = DK / 32, DT = DV / 16;
  const int lane = threadIdx.x & 63, li = lane & 15, g = lane >> 4;
  const int G = a.heads / a.kv_heads, j = tile * 16 + li;
  const int head = kvh * G + min(j, G - 1);
  int n;
  const bf16_t* arena;
  if (a.direct.used) { n = a.direct.n[b & 3]; arena = a.direct.base[b & 3]; }
  else { const int slot = a.slots[b]; n = a.kv_len[slot] + 1; arena = a.kv_base[slot]; }
  const int ntile = (n + 31) >> 5, per = (ntile + a.nsplit - 1) / a.nsplit, t0 = split * per, t1 = min(ntile, t0 + per);
  if (t0 >= t1) return;                                              // the merge knows which splits exist
  const bf16_t* kb = arena + a.k_off + (size_t)kvh * a.lmax * DK;
  const bf16_t* vb = arena + a.v_off + (size_t)kvh * a.lmax * DV;
  const float slope = a.slope ? a.slope[head] : 0.f;
  u32x4 qf[KS], knew[NEW ? KS : 1];
  bf16_t vnew[NEW ? DT : 1];
  const bool owner = NEW && t1 == ntile;                             // of the new token's key and value
  if (NEW) {
    // fragments straight from the projection: lane (head li, g) holds channels 32 k + 8 g .. of its head, the four g of a head share its norm
    const float* row = in.part + (size_t)b * in.ldn;
    const float temp = 1.f + in.temp_coef * logf((float)(n / in.temp_every) + 1.f);      // position n - 1
    auto normed = [&](const float* src, const bf16_t* w, float f, u32x4* dst) {
      f32x4 x[2 * KS];
      u32x4 wv[KS];
      float ss = 0.f;
#pragma unroll
      for (int k = 0; k < KS; ++k) {
        x[2 * k] = *reinterpret_cast<const f32x4*>(src + k * 32 + g * 8);
        x[2 * k + 1] = *reinterpret_cast<const f32x4*>(src + k * 32 + g * 8 + 4);
        wv[k] = ld16(w + k * 32 + g * 8);
      }
#pragma unroll
      for (int k = 0; k < 2 * KS; ++k) ss += (x[k][0] * x[k][0] + x[k][1] * x[k][1]) + (x[k][2] * x[k][2] + x[k][3] * x[k][3]);
      ss += __shfl_xor(ss, 16, 64);
      ss += __shfl_xor(ss, 32, 64);
      const float r = f / sqrtf(ss / (float)in.dim + in.eps);
#pragma unroll
      for (int k = 0; k < KS; ++k) {
        const u32x2 lo = pack4(x[2 * k] * r * unpack4((u32x2){wv[k][0], wv[k][1]})), hi = pack4(x[2 * k + 1] * r * unpack4((u32x2){wv[k][2], wv[k][3]}));
        dst[k] = (u32x4){lo.x, lo.y, hi.x, hi.y};
      }
    };
    normed(row + (size_t)head * DK, in.q_norm, temp, qf);
    if (owner) {
      normed(row + (size_t)(a.heads + kvh) * DK, in.k_norm, 1.f, knew);
#pragma unroll
      for (int d = 0; d < DT; ++d) vnew[NEW ? d : 0] = f2bf(row[(size_t)(a.heads + a.kv_heads) * DK + kvh * DV + d * 16 + li]);
    }
  } else {
#pragma unroll
    for (int k = 0; k < KS; ++k) qf[k] = ld16(a.q + ((size_t)b * a.heads + head) * DK + k * 32 + g * 8);
  }
  const int krow = (li >> 2) * 8 + (li & 3);                         // row li of key tile u holds key (li / 4) 8 + 4 u + li % 4
  u32x4 kf[2][KS], vf[DT];
  auto load_k = [&](int t) {
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int k = 0; k < KS; ++k) kf[u][k] = ld16(kb + (size_t)(t * 32 + krow + 4 * u) * DK + k * 32 + g * 8);      // whole tiles of the arena are readable
  };
  auto load_v = [&](int t) {
#pragma unroll
    for (int d = 0; d < DT; ++d) vf[d] = ld16(vb + ((size_t)t * DV + d * 16 + li) * 32 + g * 8);
  };
  f32x4 o[DT];
#pragma unroll
  for (int d = 0; d < DT; ++d) o[d] = (f32x4){0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  load_k(t0);
  load_v(t0);
  for (int t = t0; t < t1; ++t) {
    if (NEW && owner && t == ntile - 1) {                            // the new token: into the operands, and -- one wave per KV head -- into the cache
      const int at = (n - 1) & 31;
#pragma unroll
      for (int u = 0; u < 2; ++u)
        if (krow + 4 * u == at) {
#pragma unroll
          for (int k = 0; k < KS; ++k) {
            kf[u][k] = knew[NEW ? k : 0];
            if (tile == 0) st16(const_cast<bf16_t*>(kb) + (size_t)(n - 1) * DK + k * 32 + g * 8, knew[NEW ? k : 0]);
          }
        }
      if (at >> 3 == g) {
        const int e = at & 7, half = (e & 1) * 16;
#pragma unroll
        for (int d = 0; d < DT; ++d) {
          const unsigned keep = ~(0xffffu << half), put = (unsigned)vnew[NEW ? d : 0] << half;
#pragma unroll
          for (int q = 0; q < 4; ++q)
            if (e >> 1 == q) vf[d][q] = (vf[d][q] & keep) | put;
          if (tile == 0) const_cast<bf16_t*>(vb)[((size_t)t * DV + d * 16 + li) * 32 + at] = vnew[NEW ? d : 0];
        }
      }
    }
    f32x4 s[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      s[u] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < KS; ++k) s[u] = mfma16(as_bf16x8(kf[u][k]), as_bf16x8(qf[k]), s[u]);
    }
    if (t + 1 < t1) load_k(t + 1);
    float mx = -INFINITY;
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = t * 32 + g * 8 + u * 4 + r;
        s[u][r] = key < n ? fmaf(s[u][r], a.scale_log2e, slope * (float)(key + 1 - n)) : -INFINITY;
        mx = fmaxf(mx, s[u][r]);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float mn = fmaxf(m, mx), alpha = __builtin_amdgcn_exp2f(m - mn);      // finite: a tile has at least one key
    m = mn;
    float p[8], sum = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) { p[e] = __builtin_amdgcn_exp2f(s[e >> 2][e & 3] - mn); sum += p[e]; }
    l = l * alpha + sum;
    const bf16x8 pf = as_bf16x8((u32x4){pack2(p[0], p[1]), pack2(p[2], p[3]), pack2(p[4], p[5]), pack2(p[6], p[7])});
#pragma unroll
    for (int d = 0; d < DT; ++d) { o[d] *= alpha; o[d] = mfma16(as_bf16x8(vf[d]), pf, o[d]); }
    if (t + 1 < t1) load_v(t + 1);
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (j >= G) return;
  const size_t at = ((size_t)b * a.heads + head) * a.nsplit + split;
#pragma unroll
  for (int d = 0; d < DT; ++d) *reinterpret_cast<f32x4*>(a.ws_o + at * DV + d * 16 + g * 4) = o[d];
  if (g == 0) { a.ws_ml[at * 2] = m; a.ws_ml[at * 2 + 1] = l; }
}

}  // namespace lcc
