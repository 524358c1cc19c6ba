// Decode attention of grouped queries with a linear distance bias per head, head sizes 64 .. 256 (gfx950).  The prefill form is attn_mha32_kernel
// (attn32.hip, MhaArgs::grp_slot); both read the slot's K [kv head][Lmax][dim] and blocked-transposed V [kv head][Lmax / 32][vdim][32].
//     score(i, j) = (q_i . k_j) scale - slope_h (i - j),   everything of the score and the softmax in fp32
// The wave's work is gqa_decode_wave (mixer_ops.h).  Beside a recurrent mixer of common sizes it runs in the recurrence's launch, straight from the
// input projection (recurrent.hip: rec_gqa_decode).
#include <algorithm>

#include "mixer_ops.h"

namespace lcc {

template <int DK, int DV>
__global__ __launch_bounds__(64, DK + DV > 448 ? 1 : 2) void gqa_decode_kernel(GqaDecodeArgs a) {
  const int ht = (a.heads / a.kv_heads + 15) / 16;
  gqa_decode_wave<DK, DV, false>(a, GqaInArgs(), blockIdx.x, blockIdx.y / ht, blockIdx.y % ht, blockIdx.z);
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

// Merge of the splits, a wave per (row, head) -- or, many splits, a block: its threads share the splits; the blocks in front run the gated norm of the recurrent mixer beside it (one block per row and group).
constexpr int GQA_WAVE_SPLITS = 8;
static int merge_blocks(const GqaDecodeArgs& a, int nw) { return a.nsplit > GQA_WAVE_SPLITS ? a.rows * a.heads : (a.rows * a.heads + nw - 1) / nw; }
template <int NW, int MAXP>
__global__ __launch_bounds__(NW * 64) void gqa_merge_rec_norm_kernel(GqaDecodeArgs a, RecNormArgs nrm, int n_norm) {
  __shared__ float red[NW];
  if ((int)blockIdx.x < n_norm) {                      // the longer work first
    const int row = blockIdx.x / nrm.norm_groups;
    rec_norm_row<NW, MAXP>(nrm, row, (int)blockIdx.x - row * nrm.norm_groups, red);
    return;
  }
  const bool wide = a.nsplit > GQA_WAVE_SPLITS;
  const int lane = threadIdx.x & 63, item = wide ? (int)blockIdx.x - n_norm : ((int)blockIdx.x - n_norm) * NW + (int)(threadIdx.x >> 6);
  if (item >= a.rows * a.heads) return;
  const int b = item / a.heads;
  const int n = a.direct.used ? a.direct.n[b & 3] : a.kv_len[a.slots[b]] + 1;
  const int ntile = (n + 31) >> 5, per = (ntile + a.nsplit - 1) / a.nsplit, live = (ntile + per - 1) / per;
  const float* ml = a.ws_ml + (size_t)item * a.nsplit * 2;
  const float m = lane < live ? ml[lane * 2] : -INFINITY, l = lane < live ? ml[lane * 2 + 1] : 0.f;      // GQA_MAX_SPLIT = 64
  const bool on = lane * 4 < a.vdim;
  const float* op = a.ws_o + (size_t)item * a.nsplit * a.vdim + (on ? lane * 4 : 0);
  const float w = __builtin_amdgcn_exp2f(m - wave_max(m));
  const float wn = w / wave_sum(w * l);
  f32x4 o = {0.f, 0.f, 0.f, 0.f};
  if (wide) {
    __shared__ f32x4 s_o[NW * 64];
    __shared__ float s_w[GQA_MAX_SPLIT];
    const int tid = threadIdx.x, nc = a.vdim >> 2, ng = NW * 64 / nc, grp = tid / nc, c = tid - grp * nc;      // ng groups of nc threads
    if (tid < 64) s_w[tid] = wn;
    __syncthreads();
    if (grp < ng) {
      const float* at = a.ws_o + (size_t)item * a.nsplit * a.vdim + c * 4;
#pragma unroll 4
      for (int s = grp; s < live; s += ng) o += *reinterpret_cast<const f32x4*>(at + (size_t)s * a.vdim) * s_w[s];
    }
    s_o[tid] = o;
    __syncthreads();
    if (tid < nc) {
      for (int k = 1; k < min(ng, live); ++k) o += s_o[k * nc + tid];
      st8(a.out + (size_t)item * a.vdim + tid * 4, pack4(o));
    }
    return;
  }
  for (int s0 = 0; s0 < live; s0 += 8) {               // eight splits in flight; absent ones have weight 0
    f32x4 v[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = *reinterpret_cast<const f32x4*>(op + (size_t)min(s0 + i, live - 1) * a.vdim);
#pragma unroll
    for (int i = 0; i < 8; ++i) o += v[i] * (s0 + i < live ? __shfl(wn, s0 + i, 64) : 0.f);
  }
  if (on) st8(a.out + (size_t)item * a.vdim + lane * 4, pack4(o));
}
int gqa_merge(const GqaDecodeArgs& m, hipStream_t st) {
  if (m.rows <= 0) return 0;
  if (!gqa_ok(m) || m.vdim > 256 || (m.vdim & 63)) return LCC_ERR_SHAPE;
  if (!m.out) return LCC_ERR_ARG;
  gqa_merge_rec_norm_kernel<4, 1><<<dim3(merge_blocks(m, 4)), dim3(256), 0, st>>>(m, RecNormArgs(), 0);
  return 0;
}
bool rec_norm_ok(const RecNormArgs& a);
int gqa_merge_rec_norm(const GqaDecodeArgs& m, const RecNormArgs& a, hipStream_t st) {
  if (m.rows <= 0) return 0;
  if (!gqa_ok(m) || !rec_norm_ok(a) || a.rows != m.rows || m.vdim > 256 || (m.vdim & 63) || a.conv) return LCC_ERR_SHAPE;
  if (!m.out) return LCC_ERR_ARG;
  const int n_norm = a.rows * a.norm_groups;
  if (a.heads * a.vdim / a.norm_groups <= 1024) gqa_merge_rec_norm_kernel<4, 1><<<dim3(n_norm + merge_blocks(m, 4)), dim3(256), 0, st>>>(m, a, n_norm);
  else gqa_merge_rec_norm_kernel<16, 2><<<dim3(n_norm + merge_blocks(m, 16)), dim3(1024), 0, st>>>(m, a, n_norm);
  return 0;
}

}  // namespace lcc
