// Decode attention of grouped queries with a linear distance bias per head, head sizes 64 .. 256 (gfx950).  The prefill form is attn_mha32_kernel
// (attn32.hip, MhaArgs::grp_slot); both read the slot's K [kv head][Lmax][dim] and blocked-transposed V [kv head][Lmax / 32][vdim][32].
//     score(i, j) = (q_i . k_j) scale - slope_h (i - j),   everything of the score and the softmax in fp32
// One wave per (key split, KV head, 16 query heads of it, row), as attn_decode_kernel (attention.hip): a 32-key tile is two 16-key MFMA row
// tiles whose rows are dealt so that the probabilities a lane ends up with are the 8 consecutive keys its operand of the P.V product needs.
#include <algorithm>

#include "mixer_ops.h"

namespace lcc {

template <int DK, int DV>
__global__ __launch_bounds__(64, DK + DV > 448 ? 1 : 2) void gqa_decode_kernel(GqaDecodeArgs a) {
  constexpr int KS = DK / 32, DT = DV / 16;
  const int lane = threadIdx.x, li = lane & 15, g = lane >> 4;
  const int G = a.heads / a.kv_heads, ht = (G + 15) / 16;
  const int split = blockIdx.x, kvh = blockIdx.y / ht, j = (blockIdx.y - kvh * ht) * 16 + li, b = blockIdx.z;
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
  u32x4 qf[KS];
#pragma unroll
  for (int k = 0; k < KS; ++k) qf[k] = ld16(a.q + ((size_t)b * a.heads + head) * DK + k * 32 + g * 8);
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

template <int DK>
static int gqa_pick(const GqaDecodeArgs& a, hipStream_t st) {
  const int G = a.heads / a.kv_heads;
  const dim3 grid(a.nsplit, a.kv_heads * ((G + 15) / 16), a.rows);
  switch (a.vdim) {
    case 64: gqa_decode_kernel<DK, 64><<<grid, dim3(64), 0, st>>>(a); break;
    case 128: gqa_decode_kernel<DK, 128><<<grid, dim3(64), 0, st>>>(a); break;
    case 192: gqa_decode_kernel<DK, 192><<<grid, dim3(64), 0, st>>>(a); break;
    case 256: gqa_decode_kernel<DK, 256><<<grid, dim3(64), 0, st>>>(a); break;
    default: return LCC_ERR_SHAPE;
  }
  return 0;
}
static bool gqa_ok(const GqaDecodeArgs& a) {
  return a.heads >= 1 && a.kv_heads >= 1 && a.heads % a.kv_heads == 0 && a.heads <= 65535 && a.nsplit >= 1 && a.nsplit <= GQA_MAX_SPLIT && a.rows <= 65535 &&
         a.lmax >= 32 && !(a.lmax & 31) && a.slots && a.kv_len && a.ws_o && a.ws_ml && (!a.direct.used || a.rows <= 4);
}
int gqa_decode(const GqaDecodeArgs& a, hipStream_t st) {
  if (a.rows <= 0) return 0;
  if (!gqa_ok(a)) return LCC_ERR_SHAPE;
  if (!a.q || !a.kv_base) return LCC_ERR_ARG;
  switch (a.dim) {
    case 64: return gqa_pick<64>(a, st);
    case 128: return gqa_pick<128>(a, st);
    case 192: return gqa_pick<192>(a, st);
    case 256: return gqa_pick<256>(a, st);
    default: return LCC_ERR_SHAPE;
  }
}

// Merge of the splits, a wave per (row, head); the blocks behind run the gated norm of the recurrent mixer beside it (one block per row and group).
__global__ __launch_bounds__(256) void gqa_merge_rec_norm_kernel(GqaDecodeArgs a, RecNormArgs nrm, int n_norm) {
  __shared__ float red[4];
  if ((int)blockIdx.x < n_norm) {                      // the longer work first
    const int row = blockIdx.x / nrm.norm_groups;
    rec_norm_row<4>(nrm, row, (int)blockIdx.x - row * nrm.norm_groups, red);
    return;
  }
  const int lane = threadIdx.x & 63, item = ((int)blockIdx.x - n_norm) * 4 + (threadIdx.x >> 6);
  if (item >= a.rows * a.heads) return;
  const int b = item / a.heads;
  const int n = a.direct.used ? a.direct.n[b & 3] : a.kv_len[a.slots[b]] + 1;
  const int ntile = (n + 31) >> 5, per = (ntile + a.nsplit - 1) / a.nsplit, live = (ntile + per - 1) / per;
  const float* ml = a.ws_ml + (size_t)item * a.nsplit * 2;
  const float m = lane < live ? ml[lane * 2] : -INFINITY, l = lane < live ? ml[lane * 2 + 1] : 0.f;      // GQA_MAX_SPLIT = 64
  const float w = __builtin_amdgcn_exp2f(m - wave_max(m));
  const float wn = w / wave_sum(w * l);
  const float* op = a.ws_o + (size_t)item * a.nsplit * a.vdim + lane * 4;
  f32x4 o = {0.f, 0.f, 0.f, 0.f};
  const bool on = lane * 4 < a.vdim;
#pragma unroll 8
  for (int s = 0; s < live; ++s) {
    const float ws = __shfl(wn, s, 64);
    if (on) o += *reinterpret_cast<const f32x4*>(op + (size_t)s * a.vdim) * ws;
  }
  if (on) st8(a.out + (size_t)item * a.vdim + lane * 4, pack4(o));
}
int gqa_merge(const GqaDecodeArgs& m, hipStream_t st) {
  if (m.rows <= 0) return 0;
  if (!gqa_ok(m) || m.vdim > 256 || (m.vdim & 63)) return LCC_ERR_SHAPE;
  if (!m.out) return LCC_ERR_ARG;
  gqa_merge_rec_norm_kernel<<<dim3((m.rows * m.heads + 3) / 4), dim3(256), 0, st>>>(m, RecNormArgs(), 0);
  return 0;
}
bool rec_norm_ok(const RecNormArgs& a);
int gqa_merge_rec_norm(const GqaDecodeArgs& m, const RecNormArgs& a, hipStream_t st) {
  if (m.rows <= 0) return 0;
  if (!gqa_ok(m) || !rec_norm_ok(a) || a.rows != m.rows || m.vdim > 256 || (m.vdim & 63) || a.conv) return LCC_ERR_SHAPE;
  if (!m.out) return LCC_ERR_ARG;
  const int n_norm = a.rows * a.norm_groups;
  gqa_merge_rec_norm_kernel<<<dim3(n_norm + (m.rows * m.heads + 3) / 4), dim3(256), 0, st>>>(m, a, n_norm);
  return 0;
}

}  // namespace lcc
