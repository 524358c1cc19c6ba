// Device code shared by latent.hip and decode_v2.hip.
#pragma once
#include "common.h"
#include "kernels.h"

namespace lcc {

LCC_DEVICE float dyt_value(float x, float alpha, float w, float b) { return fmaf(tanhf(alpha * x), w, b); }

// One new row behind the fused input projection, by a block of NT threads: part = fp32 slabs [nsplit][rows][ldn] with the columns
//   [0, qp) query latent | [qp, qp + rp) cache latent (rp = 0: the layer reads another layer's cache) | then one gate value per head.
// Writes the normed query latent (bf16 [rows][qp]; QUERY false: its consumer norms it), the normed cache latent straight into the slot's
// arena, and the sigmoid gates (fp32).  The padding columns are exact zeros (zero weight rows), so the sums of squares run over the padded
// widths and divide by the real ones.  red: 2 * NT / 64 floats of LDS.
template <int NT, bool QUERY>
LCC_DEVICE void latent_row(const LatentInArgs& a, int row, float* red) {
  constexpr int NW = NT / 64;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const size_t slab = (size_t)a.rows * a.ldn;
  const float* src = a.part + (size_t)row * a.ldn;
  auto at = [&](int c) {
    f32x4 v = *reinterpret_cast<const f32x4*>(src + c);
    for (int s = 1; s < a.nsplit; ++s) v += *reinterpret_cast<const f32x4*>(src + s * slab + c);
    return v;
  };
  bf16_t* dst = nullptr;
  if (a.rp > 0) {
    const int slot = a.tok_stream[row];
    dst = a.kv_base[slot] + a.kv_off + (size_t)(a.tok_pos ? a.tok_pos[row] : a.kv_len[slot]) * a.rp;
  }
  float sq = 0.f, sk = 0.f;
  if (QUERY)
    for (int c = tid * 4; c < a.qp; c += NT * 4) { const f32x4 v = at(c); sq += (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]); }
  for (int c = tid * 4; c < a.rp; c += NT * 4) { const f32x4 v = at(a.qp + c); sk += (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]); }
  sq = wave_sum(sq); sk = wave_sum(sk);
  if (lane == 0) { red[wave] = sq; red[NW + wave] = sk; }
  for (int h = tid; h < a.heads; h += NT) {
    float z = src[a.qp + a.rp + h];
    for (int s = 1; s < a.nsplit; ++s) z += src[s * slab + a.qp + a.rp + h];
    a.gate[(size_t)row * a.heads + h] = 1.f / (1.f + expf(-z));
  }
  __syncthreads();
  sq = 0.f; sk = 0.f;
#pragma unroll
  for (int w = 0; w < NW; ++w) { sq += red[w]; sk += red[NW + w]; }
  auto put = [&](bf16_t* to, const bf16_t* norm, int c, f32x4 v, float inv) {
    const u32x2 w = ld8(norm + c);
    st8(to + c, (u32x2){pack2(v[0] * inv * lo2f(w.x), v[1] * inv * hi2f(w.x)), pack2(v[2] * inv * lo2f(w.y), v[3] * inv * hi2f(w.y))});
  };
  if (QUERY) {
    const float iq = 1.f / sqrtf(sq / (float)a.q_rank + a.eps);
    for (int c = tid * 4; c < a.qp; c += NT * 4) put(a.cq + (size_t)row * a.qp, a.q_norm, c, at(c), iq);
  }
  const float ik = a.rp > 0 ? 1.f / sqrtf(sk / (float)a.kv_rank + a.eps) : 0.f;
  for (int c = tid * 4; c < a.rp; c += NT * 4) put(dst, a.kv_norm, c, at(a.qp + c), ik);
}

}  // namespace lcc
