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
  const int slot = a.tok_stream[row], pos = a.tok_pos ? a.tok_pos[row] : a.kv_len[slot];
  bf16_t* arena = a.kv_base[slot];
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
// one (row, norm group) of the gated norm behind the recurrence, by a block of NW waves; red: NW floats of LDS
template <int NW>
LCC_DEVICE void rec_norm_row(const RecNormArgs& a, int row, int grp, float* red) {
  const int tid = threadIdx.x, inner = a.heads * a.vdim, gs = inner / a.norm_groups, nt = NW * 64;
  const size_t slab = (size_t)a.rows * a.ldn;
  const float* y = a.y + (size_t)row * a.heads * a.ep;
  const size_t gate = (size_t)row * a.ldn + a.gate_col;
  bf16_t* out = a.out + (size_t)row * a.ld;
  auto gate1 = [&](int c) {
    float z = a.part[gate + c];
    for (int s = 1; s < a.nsplit; ++s) z += a.part[s * slab + gate + c];
    return z;
  };
  const int lo = grp * gs, hi = lo + gs;
  float ss = 0.f;
  if (((a.vdim | gs) & 3) == 0) {                      // pieces of 4 channels stay inside a head and a group
    for (int r = lo + tid * 4; r < hi; r += nt * 4) {
      const int h = r / a.vdim, c = h * a.ep + r - h * a.vdim;
      f32x4 v = *reinterpret_cast<const f32x4*>(y + c);
      if (a.gate_first) v *= silu4(slab_sum4(a.part, a.nsplit, slab, gate + c));
      ss += (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]);
    }
    const float inv = 1.f / sqrtf(block_sum<NW>(ss, red) / (float)gs + a.eps);
    for (int r = lo + tid * 4; r < hi; r += nt * 4) {
      const int h = r / a.vdim, c = h * a.ep + r - h * a.vdim;
      f32x4 v = *reinterpret_cast<const f32x4*>(y + c);
      const f32x4 g = slab_sum4(a.part, a.nsplit, slab, gate + c), w = unpack4(ld8(a.w + r));
      if (a.gate_first) v = v * silu4(g) * inv * w;
      else v = v * inv * w * (f32x4){sigmoid_f(g[0]), sigmoid_f(g[1]), sigmoid_f(g[2]), sigmoid_f(g[3])};
      st8(out + r, pack4(v));
    }
  } else {
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

}  // namespace lcc
