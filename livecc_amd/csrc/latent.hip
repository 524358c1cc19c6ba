// Latent attention without positions (gfx950).  Per token and owning layer the cache holds ONE normed vector c of `rank` values
// ([Lmax][rank] bf16 per slot, rank padded to a multiple of 64 with zeros); every head's keys and values are linear maps of it:
//     k_h = Uk_h c,  v_h = Uv_h c,  score = (q_h . k_h) scale
// Two evaluations of the same sums:
//   * prefill: k and v of every visible key are formed by two GEMMs per layer and the attention is an ordinary multi-head one
//     (attn32.hip: attn_mha32_kernel; attn_mha_rows_kernel here for head sizes above 128) -- per (query, key, head) dim + vdim products;
//   * decode: the key map moves to the query, a_h = Uk_h^T q_h, so that score = (a_h . c) scale and all heads share the cached vector; the
//     weighted sum of c is mapped through Uv_h once per token -- 2 rank products per (key, head), and the only HBM traffic per key is c.
// The query and key norms, the scores, the softmax and the gates are fp32; matrix operands are bf16 with fp32 accumulation.
#include <algorithm>
#include <cstdlib>

#include "common.h"
#include "kernels.h"
#include "latent_ops.h"

namespace lcc {

// ------------------------------------------------------------------------------------------------------------------------------
// One block per new row behind the fused input projection: part = fp32 slabs [nsplit][rows][ldn] with the columns
//   [0, qp) query latent | [qp, qp + rp) cache latent (rp = 0: the layer reads another layer's cache) | then one gate value per head.
// Writes the normed query latent (bf16 [rows][qp]), the normed cache latent straight into the slot's arena, and the sigmoid gates (fp32).
// The padding columns are exact zeros (zero weight rows), so the sums of squares run over the padded widths and divide by the real ones.
// ------------------------------------------------------------------------------------------------------------------------------
__global__ __launch_bounds__(256) void latent_norm_append_kernel(LatentInArgs a) {
  __shared__ float red[8];
  latent_row<256, true>(a, blockIdx.x, red);
}
int latent_norm_append(const LatentInArgs& a, hipStream_t st) {
  if (a.rows <= 0) return 0;
  if ((a.qp & 63) || a.qp <= 0 || (a.rp & 63) || a.rp < 0 || a.nsplit < 1 || (a.ldn & 3) || a.ldn < a.qp + a.rp + a.heads) return LCC_ERR_SHAPE;
  if (!a.part || !a.q_norm || !a.cq || !a.gate || a.q_rank < 1) return LCC_ERR_ARG;
  if (a.rp > 0 && (!a.kv_norm || !a.tok_stream || (!a.tok_pos && !a.kv_len) || !a.kv_base || a.kv_rank < 1)) return LCC_ERR_ARG;
  latent_norm_append_kernel<<<dim3(a.rows), dim3(256), 0, st>>>(a);
  return 0;
}

// ------------------------------------------------------------------------------------------------------------------------------
// Prefill: the visible latents of the call's streams, back to back.  16-row tiles (slot, first key, keys of the stream): every stream starts
// at a multiple of 32 rows and is zero-filled up to the next one.  Written twice: row-major [rows][rp] (A operand of the key GEMM) and in
// MFMA fragment order (the "weight" operand of the transposed value GEMM).
// ------------------------------------------------------------------------------------------------------------------------------
__global__ __launch_bounds__(256) void latent_gather_kernel(bf16_t* const* __restrict__ kv_base, size_t kv_off, int rp,
                                                            const int32_t* __restrict__ tile_slot, const int32_t* __restrict__ tile_key0,
                                                            const int32_t* __restrict__ tile_nkeys, bf16_t* __restrict__ rows_out,
                                                            bf16_t* __restrict__ frag_out, int64_t pieces) {
  const int per_tile = rp * 2;                 // 16-byte pieces of a 16-row tile
  for (int64_t p = (int64_t)blockIdx.x * 256 + threadIdx.x; p < pieces; p += (int64_t)gridDim.x * 256) {
    const int rt = (int)(p / per_tile), q = (int)(p - (int64_t)rt * per_tile);
    const int kb = q >> 6, g = (q >> 4) & 3, r = q & 15;
    const int key = tile_key0[rt] + r, col = kb * 32 + g * 8;
    u32x4 v = {0u, 0u, 0u, 0u};
    if (key < tile_nkeys[rt]) v = ld16(kv_base[tile_slot[rt]] + kv_off + (size_t)key * rp + col);
    st16(rows_out + ((size_t)rt * 16 + r) * rp + col, v);
    st16(frag_out + (size_t)p * 8, v);
  }
}
int latent_gather(bf16_t* const* kv_base, size_t kv_off, int rp, const int32_t* tile_slot, const int32_t* tile_key0, const int32_t* tile_nkeys,
                  int n_tiles, bf16_t* rows_out, bf16_t* frag_out, hipStream_t st) {
  if (n_tiles <= 0) return 0;
  if (rp <= 0 || (rp & 63)) return LCC_ERR_SHAPE;
  const int64_t pieces = (int64_t)n_tiles * rp * 2;
  latent_gather_kernel<<<dim3((unsigned)std::min<int64_t>((pieces + 255) / 256, 8192)), dim3(256), 0, st>>>(kv_base, kv_off, rp, tile_slot, tile_key0, tile_nkeys,
                                                                                                      rows_out, frag_out, pieces);
  return 0;
}

// ------------------------------------------------------------------------------------------------------------------------------
// Causal multi-head attention for head sizes the MFMA kernel does not serve: one block per (row, head), 256 keys at a time, one key per
// thread for the scores and one channel per thread for the values.
// ------------------------------------------------------------------------------------------------------------------------------
__global__ __launch_bounds__(256) void attn_mha_rows_kernel(MhaArgs a) {
  __shared__ float s_p[256], red[4];
  extern __shared__ float s_qf[];
  const int row = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  // the group of this row
  int lo = 0, hi = a.n_groups - 1;
  while (lo < hi) { const int mid = (lo + hi + 1) >> 1; if (a.grp_q0[mid] <= row) lo = mid; else hi = mid - 1; }
  const int nkeys = a.grp_pos0[lo] + (row - a.grp_q0[lo]) + 1;
  const int ldq = a.heads * a.dim;
  const bf16_t *kbase, *vbase;                         // key i: row i of kbase (pitch ldk); value: tile i / 32 (pitch vtile), channel d (pitch ldv)
  const bool slots = a.grp_slot != nullptr;
  const int ldk = slots ? a.dim : ldq, ldv = slots ? 32 : a.ldv;
  const size_t vtile = slots ? (size_t)a.vdim * 32 : 32;
  if (slots) {
    const bf16_t* arena = a.kv_base[a.grp_slot[lo]];
    const int kvh = h / (a.heads / a.kv_heads);
    kbase = arena + a.k_off + (size_t)kvh * a.lmax * a.dim;
    vbase = arena + a.v_off + (size_t)kvh * a.lmax * a.vdim;
  } else {
    kbase = a.k + (size_t)a.grp_key0[lo] * ldq + h * a.dim;
    vbase = a.vt + (size_t)h * a.vdim * a.ldv + a.grp_key0[lo];
  }
  const float slope = a.slope ? a.slope[h] : 0.f;
  for (int d = tid; d < a.dim; d += 256) s_qf[d] = bf2f(a.q[(size_t)row * ldq + h * a.dim + d]);
  __syncthreads();
  float m = -INFINITY, l = 0.f, o[4] = {0.f, 0.f, 0.f, 0.f};        // vdim <= 1024
  for (int k0 = 0; k0 < nkeys; k0 += 256) {
    const int key = k0 + tid;
    float s = -INFINITY;
    if (key < nkeys) {
      const bf16_t* kp = kbase + (size_t)key * ldk;
      float acc = 0.f;
      for (int d = 0; d < a.dim; d += 8) {
        const u32x4 v = ld16(kp + d);
#pragma unroll
        for (int e = 0; e < 4; ++e) acc = fmaf(s_qf[d + 2 * e], lo2f(v[e]), fmaf(s_qf[d + 2 * e + 1], hi2f(v[e]), acc));
      }
      s = fmaf(acc, a.scale_log2e, slope * (float)(key + 1 - nkeys));
    }
    const float wm = wave_max(s);
    if (lane == 0) red[wave] = wm;
    __syncthreads();
    const float mn = fmaxf(fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])), m);
    const float alpha = exp2f(m - mn), p = exp2f(s - mn);           // s = -inf -> 0
    m = mn;
    s_p[tid] = p;
    __syncthreads();
    const float ws = wave_sum(p);
    if (lane == 0) red[wave] = ws;
    __syncthreads();
    l = l * alpha + (red[0] + red[1]) + (red[2] + red[3]);
    const int n = min(256, nkeys - k0);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int d = tid + 256 * j;
      if (d < a.vdim) {
        const bf16_t* vp = vbase + (size_t)(k0 >> 5) * vtile + (size_t)d * ldv;
        float acc = 0.f;
        for (int i = 0; i < n; ++i) acc = fmaf(s_p[i], bf2f(vp[(size_t)(i >> 5) * vtile + (i & 31)]), acc);
        o[j] = o[j] * alpha + acc;
      }
    }
    __syncthreads();
  }
  const float f = (a.gate ? a.gate[(size_t)row * a.heads + h] : 1.f) / l;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int d = tid + 256 * j;
    if (d < a.vdim) a.out[(size_t)row * a.ldo + h * a.vdim + d] = f2bf(o[j] * f);
  }
}
static int mha_rows(const MhaArgs& a, hipStream_t st) {
  attn_mha_rows_kernel<<<dim3(a.rows, a.heads), dim3(256), (size_t)a.dim * 4, st>>>(a);
  return 0;
}
int attn_mha(const MhaArgs& a, hipStream_t st) {
  if (a.rows <= 0 || a.n_groups <= 0) return 0;
  if (a.heads < 1 || a.dim < 8 || (a.dim & 7) || a.dim > 8192 || a.vdim < 1 || a.vdim > 1024 || (!a.grp_slot && (a.ldv & 31)) || (a.ldo & 3)) return LCC_ERR_SHAPE;
  if (!a.q || !a.out || !a.grp_q0 || !a.grp_nq || !a.grp_pos0) return LCC_ERR_ARG;
  if (a.grp_slot) {
    if (!a.kv_base || a.lmax < 32 || (a.lmax & 31) || a.kv_heads < 1 || a.heads % a.kv_heads) return LCC_ERR_SHAPE;
  } else if (!a.k || !a.vt || !a.grp_key0 || a.slope) return LCC_ERR_ARG;
  if ((a.dim == 64 || a.dim == 128) && (a.vdim == 64 || a.vdim == 128)) return attn_mha32_launch(a, st);
  return mha_rows(a, st);
}

// ------------------------------------------------------------------------------------------------------------------------------
// Decode, step 1: a_h = Uk_h^T q_h for every head and row.  q arrives as the fp32 slabs of the query up-projection; the block's 16 rows are
// summed and rounded once.  grid (rank / 64, heads, row groups); wave w owns 16 rank rows; D'[r][row]: a lane stores 4 consecutive r.
// ------------------------------------------------------------------------------------------------------------------------------
__global__ __launch_bounds__(256) void latent_absorb_kernel(const float* __restrict__ q_part, int nsplit, int rows, int heads, int dim,
                                                            const bf16_t* __restrict__ ukt, int rp, bf16_t* __restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) bf16_t s_q[];       // [16][dim + 8]
  const int h = blockIdx.y, b0 = blockIdx.z * 16, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, li = lane & 15, g = lane >> 4;
  const int pitch = dim + 8, ldq = heads * dim, K32 = dim >> 5;
  const size_t slab = (size_t)rows * ldq;
  const int rt = h * (rp >> 4) + blockIdx.x * 4 + wave;              // 16-row tile of the stacked Uk^T
  const bf16_t* wp = ukt + (size_t)rt * K32 * 512 + lane * 8;
  u32x4 w0 = ld16(wp), w1 = ld16(wp + 512);                          // dim is a multiple of 64: in flight while q is summed
  const int nrow = min(16, rows - b0);
  for (int i = tid * 4; i < nrow * dim; i += 1024) {
    const int r = i / dim, d = i - r * dim;
    const float* p = q_part + (size_t)(b0 + r) * ldq + h * dim + d;
    f32x4 v = *reinterpret_cast<const f32x4*>(p);
    for (int s = 1; s < nsplit; ++s) v += *reinterpret_cast<const f32x4*>(p + s * slab);
    st8(s_q + r * pitch + d, (u32x2){pack2(v[0], v[1]), pack2(v[2], v[3])});
  }
  __syncthreads();
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  const bf16_t* xq = s_q + min(li, nrow - 1) * pitch + g * 8;
  for (int k = 0; k < K32; k += 2) {
    acc = mfma16(as_bf16x8(w0), as_bf16x8(ld16(xq + k * 32)), acc);
    acc = mfma16(as_bf16x8(w1), as_bf16x8(ld16(xq + k * 32 + 32)), acc);
    if (k + 2 < K32) { w0 = ld16(wp + (size_t)(k + 2) * 512); w1 = ld16(wp + (size_t)(k + 3) * 512); }
  }
  if (li < nrow)
    st8(out + ((size_t)(b0 + li) * heads + h) * rp + (blockIdx.x * 4 + wave) * 16 + g * 4, (u32x2){pack2(acc[0], acc[1]), pack2(acc[2], acc[3])});
}
int latent_absorb(const float* q_part, int nsplit, int rows, int heads, int dim, const bf16_t* ukt, int rp, bf16_t* out, hipStream_t st) {
  if (rows <= 0) return 0;
  if (nsplit < 1 || heads < 1 || (dim & 63) || dim < 64 || dim > 1024 || (rp & 63) || rp < 64) return LCC_ERR_SHAPE;
  if (!q_part || !ukt || !out) return LCC_ERR_ARG;
  latent_absorb_kernel<<<dim3(rp / 64, heads, (rows + 15) / 16), dim3(256), (size_t)16 * (dim + 8) * 2, st>>>(q_part, nsplit, rows, heads, dim, ukt, rp, out);
  return 0;
}

// ------------------------------------------------------------------------------------------------------------------------------
// Decode, step 2: attention over the cached latents, all heads of a row together.  rank = 64 RT.
// Block = quads of 4 waves, one quad per 16 heads; 64 keys per iteration, staged once for all quads by LDS-DMA, double buffered.  Per iteration a wave multiplies its 16 keys with its quad's 16 queries
// (S^T[key][head]: a lane owns 4 keys of one head), the quad agrees on the new maxima through LDS, and then each wave adds
// C^T . P^T for its quarter of the channels (O^T[channel][head]: again one head per lane, so the rescale factor is lane-local).  The
// C^T operand -- 8 keys of one channel per lane -- comes out of the same LDS image through ds_read_b64_tr_b16, which transposes 4 x 16
// 16-bit blocks: in a group of 16 lanes, lane l supplies 4 consecutive channels of key l / 4 and receives channel l of 4 consecutive keys.
// grid (splits, rows, head groups); partial (O, m, l) of every split as fp32.
// ------------------------------------------------------------------------------------------------------------------------------
typedef __attribute__((ext_vector_type(4))) short s16x4;
LCC_DEVICE u32x2 lds_tr4x16(const void* p) {
  return __builtin_bit_cast(u32x2, __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)(p)));
}
// LDS image of a key tile: rows of RT * 8 16-byte chunks, chunk c of key k at slot c ^ latent_swizzle(k).  The low three bits only: a DMA
// instruction copies whole 128-byte lines (1 KB contiguous at rank 512).  Eight consecutive keys get eight different slots (score operand:
// one chunk of 16 keys) and keys 4 i .. 4 i + 3 get disjoint slot PAIRS (value operand: two chunks of 4 keys), so both reads spread the banks.
LCC_DEVICE int latent_swizzle(int key) { return ((key & 3) << 1) | ((key >> 2) & 1); }
constexpr int LATENT_PP = 72;      // pitch of a head's 64 probabilities in LDS (16-byte aligned, spreads the banks)

template <int RT, int NSTAGE>
__global__ __launch_bounds__(RT > 12 ? 256 : RT >= 6 ? 512 : 1024) void latent_attn_decode_kernel(LatentDecodeArgs a) {
  constexpr int RP = RT * 64, KB = RT * 2, NP = 4 * KB;              // channels, 32-channel blocks, pieces per 64-key tile
  constexpr int PF = RT == 8 ? 8 : (KB < 4 || RT > 12 ? 2 : 4), PV = RT == 8 ? 6 : (KB < 4 || RT > 12 ? 2 : 4);      // fragments read ahead
  extern __shared__ __attribute__((aligned(16))) u32x4 lmem[];       // NSTAGE x NP pieces, then P, then the statistics
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), li = lane & 15, g = lane >> 4;
  const int quad = wave >> 2, wq = wave & 3, nw = blockDim.x >> 6, nquad = nw >> 2;
  bf16_t* s_p = reinterpret_cast<bf16_t*>(lmem + NSTAGE * NP * 64) + quad * 16 * LATENT_PP;
  float* s_m = reinterpret_cast<float*>(reinterpret_cast<bf16_t*>(lmem + NSTAGE * NP * 64) + nquad * 16 * LATENT_PP) + quad * 64;
  const int split = blockIdx.x, b = blockIdx.y;
  const int head = (blockIdx.z * nquad + quad) * 16 + li;
  int n;                                                             // cached keys and the token of this step
  const bf16_t* arena;
  if (a.direct.used) { n = a.direct.n[b & 3]; arena = a.direct.base[b & 3]; }       // by value: no dependent loads in front of the first tile
  else { const int slot = a.slots[b]; n = a.kv_len[slot] + 1; arena = a.kv_base[slot]; }
  // split s takes the tiles s, s + nsplit, ..: the blocks of a row read neighbouring tiles at any time, so the memory channels share the load
  const int ntile = (n + 63) >> 6, tb = split, te = ntile, step = a.nsplit;
  if (tb >= te) return;                                              // the merge knows which splits exist
  const bf16_t* cbase = arena + a.kv_off;

  auto issue = [&](int t, int stage) {
    const bf16_t* src = cbase + (size_t)t * 64 * RP;
    for (int p = wave; p < NP; p += nw) {
      const int u = p * 64 + lane, key = u / (RT * 8), slot = u - key * (RT * 8);          // 16-byte units of the tile image
      glds16(src + key * RP + (slot ^ latent_swizzle(key)) * 8, lds_addr(lmem + (stage * NP + p) * 64));
    }
  };
  f32x4 o[RT];
#pragma unroll
  for (int j = 0; j < RT; ++j) o[j] = (f32x4){0.f, 0.f, 0.f, 0.f};
  float m_run = -INFINITY, l_run = 0.f;

  issue(tb, 0);
  u32x4 qf[KB];                                                      // B operand: q[head][32 ks + 8 g ..]
  if (NSTAGE == 2) {
    // the quads' queries come through the second stage, copied like a key tile (fragment-shaped loads of 16 rows x 64 bytes by every wave
    // took longer than the first key tile); the second tile is issued behind the first iteration's barrier
    for (int p = wave; p < nquad * KB; p += nw) {
      const int u = p * 64 + lane, r = u / (RT * 8), slot = u - r * (RT * 8);
      const int hr = min((int)(blockIdx.z * nquad) * 16 + r, a.heads - 1);
      glds16(a.q + ((size_t)b * a.heads + hr) * RP + (slot ^ latent_swizzle(r)) * 8, lds_addr(lmem + (NP + p) * 64));
    }
  } else {
    const bf16_t* qp = a.q + ((size_t)b * a.heads + min(head, a.heads - 1)) * RP + g * 8;
#pragma unroll
    for (int ks = 0; ks < KB; ++ks) qf[ks] = ld16(qp + ks * 32);
  }
  int stage = 0;
  for (int t = tb; t < te; t += step, stage ^= NSTAGE - 1) {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    if (NSTAGE == 1 && t == tb) {                                    // the queries have landed too (common.h: glds16)
#pragma unroll
      for (int ks = 0; ks < KB; ++ks) settle_load(qf[ks]);
    }
    __syncthreads();                                                 // tile t is complete; everyone is done with the tile before
    if (NSTAGE == 2 && t == tb) {
#pragma unroll
      for (int ks = 0; ks < KB; ++ks) qf[ks] = lmem[NP * 64 + (quad * 16 + li) * (RT * 8) + ((ks * 4 + g) ^ latent_swizzle(li))];
    }
    if (NSTAGE == 2 && t != tb && t + step < te) issue(t + step, stage ^ 1);
    const u32x4* cs = lmem + stage * NP * 64;
    // fragment reads run PF steps ahead of their MFMAs (issue order pinned: hipcc otherwise waits for every read), two accumulator chains
    f32x4 s = {0.f, 0.f, 0.f, 0.f}, s2 = {0.f, 0.f, 0.f, 0.f};
    {
      bf16x8 cf[PF];
      const u32x4* krow = cs + (wq * 16 + li) * (RT * 8);
      auto key_operand = [&](int ks) { return as_bf16x8(krow[(ks * 4 + g) ^ latent_swizzle(li)]); };
#pragma unroll
      for (int i = 0; i < PF; ++i) cf[i] = key_operand(i);
#pragma unroll
      for (int ks = 0; ks < KB; ++ks) {
        if (ks & 1) s2 = mfma16(cf[ks % PF], as_bf16x8(qf[ks]), s2); else s = mfma16(cf[ks % PF], as_bf16x8(qf[ks]), s);
        if (ks + PF < KB) cf[ks % PF] = key_operand(ks + PF);
      }
      __builtin_amdgcn_sched_group_barrier(0x100, PF, 0);
#pragma unroll
      for (int ks = 0; ks < KB; ++ks) {
        __builtin_amdgcn_sched_group_barrier(0x008, 1, 0);
        if (ks + PF < KB) __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);
      }
    }
    s += s2;
    const int k0 = t * 64 + wq * 16 + g * 4;
#pragma unroll
    for (int r = 0; r < 4; ++r) s[r] = k0 + r < n ? s[r] * a.scale_log2e : -INFINITY;
    float mx = fmaxf(fmaxf(s[0], s[1]), fmaxf(s[2], s[3]));
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    if (g == 0) s_m[wq * 16 + li] = mx;
    __syncthreads();
    if (NSTAGE == 2 && t == tb && t + step < te) issue(t + step, 1);       // every wave holds its queries
    const float m_new = fmaxf(fmaxf(fmaxf(s_m[li], s_m[16 + li]), fmaxf(s_m[32 + li], s_m[48 + li])), m_run);   // finite: a tile has >= 1 key
    const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
    m_run = m_new;
    float p[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) p[r] = __builtin_amdgcn_exp2f(s[r] - m_new);
    l_run = l_run * alpha + ((p[0] + p[1]) + (p[2] + p[3]));
    st8(s_p + li * LATENT_PP + wq * 16 + g * 4, (u32x2){pack2(p[0], p[1]), pack2(p[2], p[3])});
    __syncthreads();
    {
      bf16x8 pf[2], cf[PV];
      // C^T operand i = 2 j + ks: channels of step j, keys 32 ks ..; this lane supplies 4 channels of keys 8 g + li / 4 (+ 4) of the step
      auto operand = [&](int i) {
        const int j = i >> 1, ks = i & 1, r = wq * (16 * RT) + j * 16 + (li & 3) * 4, key = ks * 32 + g * 8 + (li >> 2);
        const char* at = reinterpret_cast<const char*>(cs) + key * (RT * 128) + (r & 7) * 2;
        const int sl = ((r >> 3) ^ latent_swizzle(key)) * 16;        // of key + 4: the low bit flips
        const u32x2 lo = lds_tr4x16(at + sl), hi = lds_tr4x16(at + 4 * (RT * 128) + (sl ^ 16));
        return as_bf16x8((u32x4){lo.x, lo.y, hi.x, hi.y});
      };
      pf[0] = as_bf16x8(ld16(s_p + li * LATENT_PP + g * 8)); pf[1] = as_bf16x8(ld16(s_p + li * LATENT_PP + 32 + g * 8));
#pragma unroll
      for (int i = 0; i < PV; ++i) cf[i] = operand(i);
#pragma unroll
      for (int j = 0; j < RT; ++j) o[j] *= alpha;
#pragma unroll
      for (int i = 0; i < KB; ++i) {
        o[i >> 1] = mfma16(cf[i % PV], pf[i & 1], o[i >> 1]);
        if (i + PV < KB) cf[i % PV] = operand(i + PV);
      }
      __builtin_amdgcn_sched_group_barrier(0x100, 2 + 2 * PV, 1);
#pragma unroll
      for (int i = 0; i < KB; ++i) {
        __builtin_amdgcn_sched_group_barrier(0x008, 1, 1);
        if (i + PV < KB) __builtin_amdgcn_sched_group_barrier(0x100, 2, 1);
      }
    }
    if (NSTAGE == 1 && t + step < te) { __syncthreads(); issue(t + step, 0); }
  }
  // the quad's denominators: over the lane groups of a wave, then over its four waves
  l_run += __shfl_xor(l_run, 16, 64);
  l_run += __shfl_xor(l_run, 32, 64);
  __syncthreads();
  if (g == 0) s_m[wq * 16 + li] = l_run;
  __syncthreads();
  if (head >= a.heads) return;
  const size_t pslot = ((size_t)b * a.heads + head) * a.nsplit + split;
  if (wq == 0 && g == 0) {
    a.ws_ml[pslot * 2] = m_run;
    a.ws_ml[pslot * 2 + 1] = (s_m[li] + s_m[16 + li]) + (s_m[32 + li] + s_m[48 + li]);
  }
  float* op = a.ws_o + pslot * RP + wq * (16 * RT) + g * 4;
#pragma unroll
  for (int j = 0; j < RT; ++j) *reinterpret_cast<f32x4*>(op + j * 16) = o[j];
}

template <int RT>
static void latent_decode_go(const LatentDecodeArgs& a, hipStream_t st) {
  constexpr int NSTAGE = RT > 8 ? 1 : 2, MAXQ = RT > 12 ? 1 : RT >= 6 ? 2 : 4;
  const int ht = (a.heads + 15) / 16;
  int groups = (ht + MAXQ - 1) / MAXQ;
  // while compute units are idle, fewer heads per block (the tiles then come out of the L2 for all but the first of a row's head groups)
  while (groups < ht && (long)a.nsplit * a.rows * std::min(2 * groups, ht) <= 256) groups = std::min(2 * groups, ht);
  const int quads = (ht + groups - 1) / groups;
  const size_t lds = (size_t)NSTAGE * 8 * RT * 1024 + (size_t)quads * (16 * LATENT_PP * 2 + 256);
  static DeviceOnce once;   // per instantiation
  if (once.first())
    (void)hipFuncSetAttribute((const void*)latent_attn_decode_kernel<RT, NSTAGE>, hipFuncAttributeMaxDynamicSharedMemorySize,
                              (int)((size_t)NSTAGE * 8 * RT * 1024 + (size_t)MAXQ * (16 * LATENT_PP * 2 + 256)));
  latent_attn_decode_kernel<RT, NSTAGE><<<dim3(a.nsplit, a.rows, groups), dim3(quads * 256), lds, st>>>(a);
}
int latent_attn_decode(const LatentDecodeArgs& a, hipStream_t st) {
  if (a.rows <= 0) return 0;
  if (a.heads < 1 || a.nsplit < 1 || a.nsplit > LATENT_MAX_SPLIT || a.rows > 65535) return LCC_ERR_SHAPE;
  if (!a.q || !a.slots || !a.kv_len || !a.kv_base || !a.ws_o || !a.ws_ml) return LCC_ERR_ARG;
  switch (a.rp) {      // the padded ranks (config.py: pad_kv_rank)
    case 64: latent_decode_go<1>(a, st); break;
    case 128: latent_decode_go<2>(a, st); break;
    case 192: latent_decode_go<3>(a, st); break;
    case 256: latent_decode_go<4>(a, st); break;
    case 384: latent_decode_go<6>(a, st); break;
    case 512: latent_decode_go<8>(a, st); break;
    case 768: latent_decode_go<12>(a, st); break;
    case 1024: latent_decode_go<16>(a, st); break;
    default: return LCC_ERR_SHAPE;
  }
  return 0;
}

// ------------------------------------------------------------------------------------------------------------------------------
// Decode, step 3: merge the splits, map the weighted latent through Uv_h, apply the head's gate.  One block per (head, group of rpb rows), a
// wave per 16 value channels.
// ------------------------------------------------------------------------------------------------------------------------------
// The Uv fragments are requested before the merge, which hides their latency (rank <= 512; above, in two batches).
template <int RT>
__global__ __launch_bounds__(1024) void latent_merge_uv_kernel(LatentDecodeArgs a, const bf16_t* __restrict__ uv, int vdim,
                                                               const float* __restrict__ gate, bf16_t* __restrict__ out, int ldo, int rpb, int vw) {
  constexpr int rp = RT * 64, pitch = rp + 8, KB = RT * 2, KW = KB > 16 ? KB / 2 : KB, NC = rp / 4;
  extern __shared__ __attribute__((aligned(16))) bf16_t s_o[];       // [rpb][rp + 8]
  __shared__ float s_w[16][LATENT_MAX_SPLIT];
  __shared__ f32x4 s_red[1024];
  __shared__ int s_live[16];
  const int h = blockIdx.y, b0 = blockIdx.z * rpb, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, li = lane & 15, g = lane >> 4;
  const int nt = blockDim.x, nw = nt >> 6, nrow = min(rpb, a.rows - b0);
  const int v0 = wave < vw ? (int)(blockIdx.x * vw + wave) * 16 : vdim;      // this wave's value channels
  const bf16_t* wp = uv + (size_t)(h * vdim + min(v0, vdim - 16) + li) * rp + g * 8;
  u32x4 wf[KW];
  if (v0 < vdim) {
#pragma unroll
    for (int k = 0; k < KW; ++k) wf[k] = ld16(wp + k * 32);
  }
  for (int r = wave; r < nrow; r += nw) {                            // the normalised weight of every split of a row
    const int b = b0 + r;
    const int n = a.direct.used ? a.direct.n[b & 3] : a.kv_len[a.slots[b]] + 1;
    const int live = min(a.nsplit, (n + 63) >> 6);                   // splits that ran: one per key tile at most
    const float* ml = a.ws_ml + ((size_t)b * a.heads + h) * a.nsplit * 2;
    const bool h0 = lane < live, h1 = lane + 64 < live;              // LATENT_MAX_SPLIT = 128: two per lane
    const float m0 = h0 ? ml[lane * 2] : -INFINITY, m1 = h1 ? ml[(lane + 64) * 2] : -INFINITY;
    const float l0 = h0 ? ml[lane * 2 + 1] : 0.f, l1 = h1 ? ml[(lane + 64) * 2 + 1] : 0.f;
    const float m = wave_max(fmaxf(m0, m1));
    const float e0 = __builtin_amdgcn_exp2f(m0 - m), e1 = __builtin_amdgcn_exp2f(m1 - m);
    const float inv = 1.f / wave_sum(e0 * l0 + e1 * l1);
    s_w[r][lane] = e0 * inv;
    s_w[r][lane + 64] = e1 * inv;
    if (lane == 0) s_live[r] = live;
  }
  __syncthreads();
  // weighted sum of the splits: one 4-channel piece per thread; with fewer pieces than threads several threads share a piece's splits
  const int items = nrow * NC, share = max(1, nt / items), pieces = share > 1 ? items : nt;
  for (int i0 = 0; i0 < items; i0 += pieces) {
    const int part = share > 1 ? tid / items : 0, item = i0 + (share > 1 ? tid - part * items : tid);
    const bool on = item < items && part < share;
    const int r = on ? item / NC : 0, c = (on ? item - r * NC : 0) * 4;
    f32x4 v = {0.f, 0.f, 0.f, 0.f};
    if (on) {
      const int live = s_live[r];
      const float* op = a.ws_o + ((size_t)(b0 + r) * a.heads + h) * a.nsplit * rp + c;
#pragma unroll 8
      for (int s = part; s < live; s += share) v += *reinterpret_cast<const f32x4*>(op + (size_t)s * rp) * s_w[r][s];
    }
    if (share > 1) {
      s_red[tid] = v;
      __syncthreads();
      if (on && part == 0)
        for (int p = 1; p < share; ++p) v += s_red[p * items + item];
    }
    if (on && part == 0) st8(s_o + r * pitch + c, (u32x2){pack2(v[0], v[1]), pack2(v[2], v[3])});
  }
  __syncthreads();
  if (v0 >= vdim) return;
  const bf16_t* xp = s_o + min(li, nrow - 1) * pitch + g * 8;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f}, acc2 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int k = 0; k < KB; ++k) {
    if (k & 1) acc2 = mfma16(as_bf16x8(wf[k % KW]), as_bf16x8(ld16(xp + k * 32)), acc2);
    else acc = mfma16(as_bf16x8(wf[k % KW]), as_bf16x8(ld16(xp + k * 32)), acc);
    if (k + KW < KB) wf[k % KW] = ld16(wp + (k + KW) * 32);
  }
  acc += acc2;
  if (li < nrow) {
    const float f = gate ? gate[(size_t)(b0 + li) * a.heads + h] : 1.f;
    st8(out + (size_t)(b0 + li) * ldo + h * vdim + v0 + g * 4, (u32x2){pack2(acc[0] * f, acc[1] * f), pack2(acc[2] * f, acc[3] * f)});
  }
}
int latent_merge_uv(const LatentDecodeArgs& a, const bf16_t* uv, int vdim, const float* gate, bf16_t* out, int ldo, hipStream_t st) {
  if (a.rows <= 0) return 0;
  if ((vdim & 63) || vdim < 64 || (a.rp & 63) || a.rp < 64 || a.rp > 1024 || (ldo & 3) || a.nsplit > LATENT_MAX_SPLIT || a.nsplit < 1) return LCC_ERR_SHAPE;
  if (!uv || !out || !a.ws_o || !a.ws_ml || !a.slots || !a.kv_len) return LCC_ERR_ARG;
  int rpb = 16;                                                      // rows per block: as many as still give the chip a block per CU
  while (rpb > 1 && (long)a.heads * ((a.rows + rpb - 1) / rpb) < 192) rpb >>= 1;
  const size_t lds = (size_t)rpb * (a.rp + 8) * 2;
  const int threads = rpb <= 4 ? 1024 : 512;
  // value channels of a block: all its waves', or -- few blocks -- 64 (the blocks of a head then merge the same partial sums)
  const int vw = a.heads * a.rows < 96 ? 4 : threads / 64;
  const dim3 grid((vdim / 16 + vw - 1) / vw, a.heads, (a.rows + rpb - 1) / rpb);
#define LCC_MERGE(RT) case RT * 64: latent_merge_uv_kernel<RT><<<grid, dim3(threads), lds, st>>>(a, uv, vdim, gate, out, ldo, rpb, vw); break
  switch (a.rp) {
    LCC_MERGE(1); LCC_MERGE(2); LCC_MERGE(3); LCC_MERGE(4); LCC_MERGE(6); LCC_MERGE(8); LCC_MERGE(12); LCC_MERGE(16);
    default: return LCC_ERR_SHAPE;
  }
#undef LCC_MERGE
  return 0;
}

}  // namespace lcc
