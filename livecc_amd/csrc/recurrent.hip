// Recurrent mixers with one scalar decay per head and token (linear attention with a fixed decay, state-space duality), gfx950:
//     S_t = 2^(rate dt_t) S_{t-1} + dt_t k_t v_t^T,     o_t = S_t^T q_t (+ skip v_t),          S [key][value] fp32 per head
// keys and queries may be shared by the heads of a group.  The state of a stream lives in its slot's arena.
//   * decode: one pass over the state (rec_decode_kernel), HBM-bound; input activations (and the short convolution) are part of it.
//   * prefill: chunks of 64 tokens on the matrix cores (rec_scan_kernel): inside a chunk
//         o = ((q k^T) * 2^(L_t - L_s) dt_s, s <= t) v + 2^(L_t) q S,       S <- 2^(L_end) S + k^T (2^(L_end - L_s) dt_s v)
//     with L the running sum of rate dt, so every exponent is <= 0.  Long prompts are cut into segments: their states from zero (phase 1), the
//     states they start from (phase 2, elementwise), their outputs (phase 3) -- the chip is then full whatever the number of heads.
// Decays, step sizes, running sums and the state are fp32.  Where the state or the weighted values are a matrix operand they go in as a bf16
// pair (value and remainder), so nothing of the recurrence is rounded to 16 bits beyond the projections themselves.
#include <algorithm>

#include "mixer_ops.h"

namespace lcc {

// ------------------------------------------------------------------------------------------------------------------------------
// Prefill, in front of the scan and the attention: one block per row.
// ------------------------------------------------------------------------------------------------------------------------------
// TAPS > 0: REC alone, PREP_ROWS rows per block -- a thread reads its columns of every row once and keeps the window in registers
constexpr int PREP_ROWS = 4;
template <int TAPS>
__global__ __launch_bounds__(256) void conv_prep_kernel(RecInArgs a) {
  constexpr int WIN = PREP_ROWS + TAPS - 1;
  const int row0 = blockIdx.x * PREP_ROWS, n = min(PREP_ROWS, a.rows - row0), tid = threadIdx.x, gk = a.groups * a.np, hv = a.heads * a.ep;
  const size_t slab = (size_t)a.rows * a.ldn;
  int pos[PREP_ROWS], r0[PREP_ROWS];
  const float* ring[PREP_ROWS];
#pragma unroll
  for (int i = 0; i < PREP_ROWS; ++i) {
    const int r = min(row0 + i, a.rows - 1);
    pos[i] = a.tok_pos[r]; r0[i] = a.tok_row0[r];
    ring[i] = reinterpret_cast<const float*>(a.kv_base[a.tok_stream[r]] + a.conv_off);
  }
  for (int p = ((int)blockIdx.y * 256 + tid) * 4; p < 2 * gk + hv; p += (int)gridDim.y * 1024) {
    const int col = p < gk ? a.q_col + p : p < 2 * gk ? a.k_col + p - gk : a.v_col + p - 2 * gk, ch = col - a.conv_col;
    f32x4 u[WIN], w[TAPS];
#pragma unroll
    for (int i = 0; i < WIN; ++i)
      u[i] = slab_sum4(a.part, a.nsplit, slab, (size_t)min(max(row0 + i - (TAPS - 1), 0), a.rows - 1) * a.ldn + col);
#pragma unroll
    for (int t = 0; t < TAPS; ++t) w[t] = unpack4(ld8(a.conv_w + (size_t)t * a.conv_ch + ch));
    const f32x4 bias = unpack4(ld8(a.conv_b + ch));
#pragma unroll
    for (int i = 0; i < PREP_ROWS; ++i) {
      if (i >= n) break;
      f32x4 acc = bias + w[TAPS - 1] * u[i + TAPS - 1];
#pragma unroll
      for (int back = 1; back < TAPS; ++back) {
        f32x4 x = u[i + TAPS - 1 - back];
        if (row0 + i - back < r0[i])                   // before this portion: out of the slot's ring, zero before the start
          x = back <= pos[i] ? *reinterpret_cast<const f32x4*>(ring[i] + (size_t)((pos[i] - back) % TAPS) * a.conv_ch + ch) : (f32x4){0.f, 0.f, 0.f, 0.f};
        acc += w[TAPS - 1 - back] * x;
      }
      const u32x2 o = pack4(silu4(acc));
      const size_t row = (size_t)(row0 + i);
      if (p < gk) st8(a.q + row * gk + p, o);
      else if (p < 2 * gk) st8(a.k + row * gk + p - gk, o);
      else st8(a.v + row * hv + p - 2 * gk, o);
    }
  }
  if (a.dt_col >= 0 && blockIdx.y == 0)
    for (int i = tid; i < n * a.heads; i += 256) a.dt[(size_t)row0 * a.heads + i] = rec_dt(a, row0 + i / a.heads, i % a.heads);
}
template <bool LEFT, bool REC>
__global__ __launch_bounds__(256) void mixer_prep_kernel(GqaInArgs l, RecInArgs a) {
  // blockIdx.y: few rows are spread over several blocks -- the attention's part, then shares of the recurrence's columns
  const int row = blockIdx.x, tid = threadIdx.x, part = LEFT && gridDim.y > 1 ? (int)blockIdx.y - 1 : (int)blockIdx.y, parts = LEFT && gridDim.y > 1 ? gridDim.y - 1 : gridDim.y;
  if (LEFT && blockIdx.y == 0) gqa_row<4>(l, row);
  if (!REC || part < 0) return;
  const int pos = a.tok_pos[row], r0 = a.tok_row0[row], gk = a.groups * a.np, hv = a.heads * a.ep;
  const float* ring = a.taps ? reinterpret_cast<const float*>(a.kv_base[a.tok_stream[row]] + a.conv_off) : nullptr;
  for (int p = (part * 256 + tid) * 4; p < 2 * gk + hv; p += parts * 1024) {
    f32x4 raw;
    if (p < gk) st8(a.q + (size_t)row * gk + p, pack4(rec_in4(a, row, r0, pos, ring, a.q_col + p, &raw)));
    else if (p < 2 * gk) st8(a.k + (size_t)row * gk + p - gk, pack4(rec_in4(a, row, r0, pos, ring, a.k_col + p - gk, &raw)));
    else st8(a.v + (size_t)row * hv + p - 2 * gk, pack4(rec_in4(a, row, r0, pos, ring, a.v_col + p - 2 * gk, &raw)));
  }
  if (a.dt_col >= 0 && part == 0)
    for (int h = tid; h < a.heads; h += 256) a.dt[(size_t)row * a.heads + h] = rec_dt(a, row, h);
}
static bool gqa_in_ok(const GqaInArgs& a) {
  return a.part && a.nsplit >= 1 && a.q_norm && a.k_norm && a.q && a.tok_stream && (a.tok_pos || a.kv_len) && a.kv_base && a.heads >= 1 && a.kv_heads >= 1 &&
         a.dim >= 1 && a.dim <= a.dim_pad && a.dim_pad <= 256 && !(a.dim_pad & 63) && !(a.vdim_pad & 63) && a.temp_every >= 1 && !(a.ldn & 3) &&
         a.ldn >= (a.heads + a.kv_heads) * a.dim_pad + a.kv_heads * a.vdim_pad && a.lmax >= 32 && !(a.lmax & 31);
}
static bool rec_in_ok(const RecInArgs& a) {
  const int gk = a.groups * a.np, hv = a.heads * a.ep;
  auto fits = [&](int col, int n) { return col >= 0 && !(col & 3) && col + n <= a.ldn && (a.taps == 0 || (col >= a.conv_col && col + n <= a.conv_col + a.conv_ch)); };
  return a.part && a.nsplit >= 1 && !(a.ldn & 3) && a.heads >= 1 && a.groups >= 1 && a.heads % a.groups == 0 && a.np >= 64 && !(a.np & 63) && a.np <= 256 &&
         a.ep >= 64 && !(a.ep & 63) && fits(a.q_col, gk) && fits(a.k_col, gk) && fits(a.v_col, hv) && (a.dt_col < 0 || (a.dt_bias && a.dt_col + a.heads <= a.ldn)) &&
         a.rate && a.tok_stream && a.kv_base && a.taps >= 0 && (a.taps == 0 || (a.conv_w && a.conv_b && !(a.conv_ch & 3) && a.conv_col + a.conv_ch <= a.ldn));
}
int mixer_prep(const GqaInArgs* left, const RecInArgs* rec, hipStream_t st) {
  const int rows = left ? left->rows : rec ? rec->rows : 0;
  if (rows <= 0) return 0;
  if (left && !gqa_in_ok(*left)) return LCC_ERR_SHAPE;
  if (rec && (!rec_in_ok(*rec) || (left && left->rows != rec->rows))) return LCC_ERR_SHAPE;
  if (rec && (!rec->tok_pos || !rec->tok_row0 || !rec->q || !rec->k || !rec->v || (rec->dt_col >= 0 && !rec->dt))) return LCC_ERR_ARG;
  const GqaInArgs l = left ? *left : GqaInArgs();
  const RecInArgs r = rec ? *rec : RecInArgs();
  const int cols = rec ? 2 * r.groups * r.np + r.heads * r.ep : 0, share = std::max(1, std::min((cols + 1023) / 1024, 2048 / rows));
  if (left && rec) mixer_prep_kernel<true, true><<<dim3(rows, share > 1 ? share + 1 : 1), dim3(256), 0, st>>>(l, r);
  else if (left) mixer_prep_kernel<true, false><<<dim3(rows), dim3(256), 0, st>>>(l, r);
  else if (r.taps == 4 && rows >= 64) conv_prep_kernel<4><<<dim3((rows + PREP_ROWS - 1) / PREP_ROWS, std::min((cols + 1023) / 1024, share * PREP_ROWS)), dim3(256), 0, st>>>(r);
  else mixer_prep_kernel<false, true><<<dim3(rows, share), dim3(256), 0, st>>>(l, r);
  return 0;
}

// ------------------------------------------------------------------------------------------------------------------------------
// Decode: block = (row, head, 64 value channels); thread t owns value channels 4 (t & 15) .. of the state rows t / 16, t / 16 + 16, ..
// The blocks behind them run the attention beside it (rec_gqa_decode_kernel), or only its rows: queries, keys, values (rec_decode_kernel).
// ------------------------------------------------------------------------------------------------------------------------------
template <int NT>
LCC_DEVICE void rec_decode_block(const RecInArgs& a, float* __restrict__ y) {
  constexpr int NP = NT * 64, NR = NP / 16;
  __shared__ float s_q[NP], s_k[NP];
  __shared__ __attribute__((aligned(16))) float s_v[64];
  __shared__ f32x4 s_o[4][16];
  const int vt = a.ep / 64, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int row = blockIdx.x / (a.heads * vt), rem = blockIdx.x - row * (a.heads * vt), h = rem / vt, v0 = (rem - h * vt) * 64;
  const int slot = a.tok_stream[row], grp = h / (a.heads / a.groups);
  int pos;
  bf16_t* arena;
  if (a.direct.used) { pos = a.direct.n[row & 3] - 1; arena = const_cast<bf16_t*>(a.direct.base[row & 3]); }
  else { pos = a.kv_len[slot]; arena = a.kv_base[slot]; }
  float* S = reinterpret_cast<float*>(arena + a.state_off) + (size_t)h * NP * a.ep + v0 + (tid & 15) * 4;
  const int n0 = tid >> 4;
  f32x4 st[NR];
#pragma unroll
  for (int i = 0; i < NR; ++i) st[i] = *reinterpret_cast<const f32x4*>(S + (size_t)(n0 + 16 * i) * a.ep);
  float* ring = a.taps ? reinterpret_cast<float*>(arena + a.conv_off) : nullptr;
  const bool frozen = a.done != nullptr && a.done[slot];
  for (int p = tid * 4; p < 2 * NP + 64; p += 1024) {
    const int col = p < NP ? a.q_col + grp * NP + p : p < 2 * NP ? a.k_col + grp * NP + p - NP : a.v_col + h * a.ep + v0 + p - 2 * NP;
    f32x4 raw;
    const f32x4 v = rec_in4(a, row, row, pos, ring, col, &raw);
    // position p replaces position p - taps, which no reader of this step needs; blocks that share a channel write the same value
    if (ring && !frozen) *reinterpret_cast<f32x4*>(ring + (size_t)(pos % a.taps) * a.conv_ch + col - a.conv_col) = raw;
    float* dst = p < NP ? s_q + p : p < 2 * NP ? s_k + p - NP : s_v + p - 2 * NP;
#pragma unroll
    for (int e = 0; e < 4; ++e) dst[e] = v[e];
  }
  const float dt = rec_dt(a, row, h), decay = pos > 0 ? exp2f(a.rate[h] * dt) : 0.f;
  __syncthreads();
  const f32x4 v = *reinterpret_cast<const f32x4*>(s_v + (tid & 15) * 4), dv = v * dt;
  f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int n = n0 + 16 * i;
    const f32x4 s = (pos > 0 ? st[i] * decay : (f32x4){0.f, 0.f, 0.f, 0.f}) + dv * s_k[n];      // a fresh slot's arena holds another stream's state
    o += s * s_q[n];
    if (!frozen) *reinterpret_cast<f32x4*>(S + (size_t)n * a.ep) = s;
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    o[e] += __shfl_xor(o[e], 16, 64);
    o[e] += __shfl_xor(o[e], 32, 64);
  }
  if (lane < 16) s_o[wave][lane] = o;
  __syncthreads();
  if (tid < 16) {
    f32x4 r = (s_o[0][tid] + s_o[1][tid]) + (s_o[2][tid] + s_o[3][tid]);
    if (a.skip) r += v * a.skip[h];
    *reinterpret_cast<f32x4*>(y + ((size_t)row * a.heads + h) * a.ep + v0 + tid * 4) = r;
  }
}
template <int NT>
__global__ __launch_bounds__(256) void rec_decode_kernel(RecInArgs a, GqaInArgs l, float* __restrict__ y, int n_rec) {
  if ((int)blockIdx.x >= n_rec) gqa_row<4>(l, (int)blockIdx.x - n_rec);
  else rec_decode_block<NT>(a, y);
}
// the attention beside it in the same launch: behind the n_rec blocks, four (split, KV head, head tile, row) items per block, splits fastest
template <int NT, int DK, int DV>
__global__ __launch_bounds__(256, 2) void rec_gqa_decode_kernel(RecInArgs a, GqaInArgs l, GqaDecodeArgs d, float* __restrict__ y, int n_rec) {
  if ((int)blockIdx.x < n_rec) { rec_decode_block<NT>(a, y); return; }
  const int ht = (d.heads / d.kv_heads + 15) / 16, per_row = d.nsplit * d.kv_heads * ht;
  const int item = __builtin_amdgcn_readfirstlane(((int)blockIdx.x - n_rec) * 4 + (int)(threadIdx.x >> 6));
  if (item >= d.rows * per_row) return;
  const int b = item / per_row, r = item - b * per_row, split = r % d.nsplit, hh = r / d.nsplit;
  gqa_decode_wave<DK, DV, true>(d, l, split, hh / ht, hh % ht, b);
}
bool rec_gqa_decode_ok(const RecInArgs& rec, const GqaDecodeArgs& d) {
  // up to 4 rows: the launch saved; from 8 rows on the two kernels' own occupancies are worth more (8 streams x 4096 keys: 25.7 against 28.6 us)
  return rec.rows <= 4 && rec.nsplit == 1 && rec.np <= 128 && (d.dim == 64 || d.dim == 128) && (d.vdim == 64 || d.vdim == 128);
}
int rec_gqa_decode(const RecInArgs& rec, const GqaInArgs& left, const GqaDecodeArgs& d, float* y, hipStream_t st) {
  if (rec.rows <= 0) return 0;
  if (!rec_in_ok(rec) || !gqa_in_ok(left) || !rec_gqa_decode_ok(rec, d) || left.rows != rec.rows || d.rows != rec.rows || left.nsplit != 1 || left.dim_pad != d.dim ||
      left.vdim_pad != d.vdim || left.heads != d.heads || left.kv_heads != d.kv_heads || d.nsplit < 1 || d.nsplit > GQA_MAX_SPLIT || d.lmax != left.lmax ||
      (d.direct.used && d.rows > 4))
    return LCC_ERR_SHAPE;
  if (!rec.kv_len || !y || !d.slots || !d.kv_len || !d.kv_base || !d.ws_o || !d.ws_ml) return LCC_ERR_ARG;
  const int n = rec.rows * rec.heads * (rec.ep / 64), items = d.rows * d.nsplit * d.kv_heads * ((d.heads / d.kv_heads + 15) / 16);
  const dim3 grid(n + (items + 3) / 4);
#define LCC_GO(NT)                                                                                                          \
  do {                                                                                                                      \
    if (d.dim == 64 && d.vdim == 64) rec_gqa_decode_kernel<NT, 64, 64><<<grid, dim3(256), 0, st>>>(rec, left, d, y, n);          \
    else if (d.dim == 64) rec_gqa_decode_kernel<NT, 64, 128><<<grid, dim3(256), 0, st>>>(rec, left, d, y, n);                    \
    else if (d.vdim == 64) rec_gqa_decode_kernel<NT, 128, 64><<<grid, dim3(256), 0, st>>>(rec, left, d, y, n);                   \
    else rec_gqa_decode_kernel<NT, 128, 128><<<grid, dim3(256), 0, st>>>(rec, left, d, y, n);                                    \
  } while (0)
  if (rec.np == 64) LCC_GO(1); else LCC_GO(2);
#undef LCC_GO
  return 0;
}
int rec_decode(const RecInArgs& rec, const GqaInArgs* left, float* y, hipStream_t st) {
  if (rec.rows <= 0) return 0;
  if (!rec_in_ok(rec) || (left && (!gqa_in_ok(*left) || left->rows != rec.rows))) return LCC_ERR_SHAPE;
  if (!rec.kv_len || !y) return LCC_ERR_ARG;
  const int n = rec.rows * rec.heads * (rec.ep / 64);
  const dim3 grid(n + (left ? rec.rows : 0));
  const GqaInArgs l = left ? *left : GqaInArgs();
  switch (rec.np / 64) {
    case 1: rec_decode_kernel<1><<<grid, dim3(256), 0, st>>>(rec, l, y, n); break;
    case 2: rec_decode_kernel<2><<<grid, dim3(256), 0, st>>>(rec, l, y, n); break;
    case 3: rec_decode_kernel<3><<<grid, dim3(256), 0, st>>>(rec, l, y, n); break;
    default: rec_decode_kernel<4><<<grid, dim3(256), 0, st>>>(rec, l, y, n); break;
  }
  return 0;
}

// ------------------------------------------------------------------------------------------------------------------------------
// Prefill scan.  Block = (segment, head, 64 value channels), 4 waves, one 64-token chunk per iteration; the next chunk's rows travel in registers
// while this one is computed.  Wave w owns the chunk's rows 16 w .. (scores, outputs) and the value channels 16 w .. of the state:
// st[i] = S[n = 16 i + 4 g + r][v = 16 w + li].  OUT: outputs; SEGMENT: the state starts at zero (OUT: at seg_state) and the end state goes
// to seg_state (OUT: nowhere); otherwise both ends are the slot's state.
// ------------------------------------------------------------------------------------------------------------------------------
template <int NT, bool OUT, bool SEGMENT>
__global__ __launch_bounds__(256, NT > 2 ? 1 : 2) void rec_scan_kernel(RecScanArgs a) {
  constexpr int NP = NT * 64, PK = NP + 8, PV = 72, NF = NP / 32, NS = NP / 16, KL = NT * 2;      // LDS pitches; fragments; state tiles; row pieces per thread
  extern __shared__ __attribute__((aligned(16))) bf16_t smem[];
  bf16_t* s_k = smem;                                  // [64][PK]
  bf16_t* s_v = s_k + 64 * PK;                         // [64][PV]
  float* s_f = reinterpret_cast<float*>(s_v + 64 * PV);      // [3][64]: L, dt, weight of a row in the chunk's end state
  bf16_t* s_q = reinterpret_cast<bf16_t*>(s_f + 192);  // [64][PK]; a wave's own rows later hold its probabilities (OUT only, as the next two)
  bf16_t* s_sh = s_q + 64 * PK;                        // [64 v][PK]: S^T, value and remainder
  bf16_t* s_sl = s_sh + 64 * PK;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, li = lane & 15, g = lane >> 4;
  const int vt = a.ep / 64, seg = blockIdx.x, h = blockIdx.y / vt, v0 = (blockIdx.y - h * vt) * 64, grp = h / (a.heads / a.groups);
  const int row0 = a.seg_row0[seg], rows = a.seg_rows[seg];
  const int ldk = a.groups * NP, ldv = a.heads * a.ep;
  const bf16_t *kp = a.k + (size_t)row0 * ldk + grp * NP, *qp = a.q + (size_t)row0 * ldk + grp * NP, *vp = a.v + (size_t)row0 * ldv + h * a.ep + v0;
  const float rate = a.rate[h], skip = OUT && a.skip ? a.skip[h] : 0.f;
  float* S = SEGMENT ? a.seg_state + ((size_t)seg * a.heads + h) * NP * a.ep : reinterpret_cast<float*>(a.kv_base[a.seg_slot[seg]] + a.state_off) + (size_t)h * NP * a.ep;
  S += v0 + wave * 16 + li;

  f32x4 st[NS];
  const bool zero = SEGMENT ? !OUT : a.seg_fresh[seg] != 0;
#pragma unroll
  for (int i = 0; i < NS; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) st[i][r] = zero ? 0.f : S[(size_t)(i * 16 + g * 4 + r) * a.ep];

  u32x4 rk[KL], rq[OUT ? KL : 1], rv[2];
  float rdt = 0.f;
  auto fetch = [&](int c0) {                           // rows past the segment read its last row; the LDS copy of k, v and dt is zero there
#pragma unroll
    for (int j = 0; j < KL; ++j) {
      const int p = j * 256 + tid, r = min(c0 + p / (NP / 8), rows - 1), c = (p % (NP / 8)) * 8;
      rk[j] = ld16(kp + (size_t)r * ldk + c);
      if (OUT) rq[OUT ? j : 0] = ld16(qp + (size_t)r * ldk + c);
    }
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int p = j * 256 + tid, r = min(c0 + (p >> 3), rows - 1);
      rv[j] = ld16(vp + (size_t)r * ldv + (p & 7) * 8);
    }
    if (wave == 0) rdt = a.dt ? a.dt[(size_t)(row0 + min(c0 + lane, rows - 1)) * a.heads + h] : 1.f;
  };
  fetch(0);
  float total = 0.f;
  for (int c0 = 0; c0 < rows; c0 += 64) {
    const int n = min(64, rows - c0);
    const u32x4 z4 = {0u, 0u, 0u, 0u};
#pragma unroll
    for (int j = 0; j < KL; ++j) {
      const int p = j * 256 + tid, r = p / (NP / 8), c = (p % (NP / 8)) * 8;
      st16(s_k + r * PK + c, r < n ? rk[j] : z4);
      if (OUT) st16(s_q + r * PK + c, rq[OUT ? j : 0]);
    }
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int p = j * 256 + tid, r = p >> 3;
      st16(s_v + r * PV + (p & 7) * 8, r < n ? rv[j] : z4);
    }
    if (wave == 0) {                                   // running sum of the log decays over the chunk
      const float dt = lane < n ? rdt : 0.f;
      float L = rate * dt;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) { const float up = __shfl_up(L, o, 64); if (lane >= o) L += up; }
      const float end = __shfl(L, 63, 64);
      s_f[lane] = L; s_f[64 + lane] = dt; s_f[128 + lane] = exp2f(end - L) * dt;
    }
    if (OUT) {
#pragma unroll
      for (int i = 0; i < NS; ++i) {                   // S^T of this wave's value channels: a lane holds 4 consecutive n
        const u32x2 hi = pack4(st[i]);
        const int at = (wave * 16 + li) * PK + i * 16 + g * 4;
        st8(s_sh + at, hi);
        st8(s_sl + at, pack4(st[i] - unpack4(hi)));
      }
    }
    __syncthreads();
    if (c0 + 64 < rows) fetch(c0 + 64);
    const float end = s_f[63];
    total += end;
    if (OUT) {
      u32x4 qf[NF];
      bf16_t* prow = s_q + (wave * 16 + li) * PK;
#pragma unroll
      for (int k = 0; k < NF; ++k) qf[k] = ld16(prow + k * 32 + g * 8);
      asm volatile("" ::: "memory");                   // the probabilities below go over these rows
      f32x4 o[4];
      float Lr[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) Lr[r] = s_f[wave * 16 + g * 4 + r];
#pragma unroll
      for (int t = 0; t < 4; ++t) {                    // q S
        f32x4 acc = {0.f, 0.f, 0.f, 0.f}, rem = acc;
#pragma unroll
        for (int k = 0; k < NF; ++k) {
          acc = mfma16(as_bf16x8(qf[k]), as_bf16x8(ld16(s_sh + (t * 16 + li) * PK + k * 32 + g * 8)), acc);
          rem = mfma16(as_bf16x8(qf[k]), as_bf16x8(ld16(s_sl + (t * 16 + li) * PK + k * 32 + g * 8)), rem);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) o[t][r] = (acc[r] + rem[r]) * exp2f(Lr[r]);
      }
      // probabilities of this wave's rows, over its own query rows (every lane holds its fragments)
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        f32x4 p = {0.f, 0.f, 0.f, 0.f};
        if (t <= wave) {
#pragma unroll
          for (int k = 0; k < NF; ++k) p = mfma16(as_bf16x8(qf[k]), as_bf16x8(ld16(s_k + (t * 16 + li) * PK + k * 32 + g * 8)), p);
          const int s = t * 16 + li;
          const float Ls = s_f[s], ds = s_f[64 + s];
#pragma unroll
          for (int r = 0; r < 4; ++r) p[r] = s <= wave * 16 + g * 4 + r ? p[r] * exp2f(Lr[r] - Ls) * ds : 0.f;
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) s_q[(wave * 16 + g * 4 + r) * PK + t * 16 + li] = f2bf(p[r]);
      }
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");      // written and read by the same wave
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        if (k == 1 && wave < 2) break;                 // keys 32 .. lie behind the rows of waves 0 and 1
        const bf16x8 pf = as_bf16x8(ld16(prow + k * 32 + g * 8));
#pragma unroll
        for (int t = 0; t < 4; ++t) {
          const bf16_t* at = s_v + (k * 32 + g * 8 + (li >> 2)) * PV + t * 16 + (li & 3) * 4;
          const u32x2 lo = lds_read_tr(at), hi = lds_read_tr(at + 4 * PV);
          o[t] = mfma16(pf, as_bf16x8((u32x4){lo.x, lo.y, hi.x, hi.y}), o[t]);
        }
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = wave * 16 + g * 4 + r;
        if (t < n) {
          float* yp = a.y + (size_t)(row0 + c0 + t) * ldv + h * a.ep + v0 + li;
#pragma unroll
          for (int j = 0; j < 4; ++j) yp[j * 16] = o[j][r] + skip * bf2f(s_v[t * PV + j * 16 + li]);
        }
      }
    }
    // the state at the chunk's end
    {
      const float de = exp2f(end);
#pragma unroll
      for (int i = 0; i < NS; ++i) st[i] *= de;
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const int s = k * 32 + g * 8;
        const bf16_t* at = s_v + (s + (li >> 2)) * PV + wave * 16 + (li & 3) * 4;
        const f32x4 w0 = *reinterpret_cast<const f32x4*>(s_f + 128 + s), w1 = *reinterpret_cast<const f32x4*>(s_f + 128 + s + 4);
        const f32x4 x0 = unpack4(lds_read_tr(at)) * w0, x1 = unpack4(lds_read_tr(at + 4 * PV)) * w1;
        const u32x2 h0 = pack4(x0), h1 = pack4(x1), l0 = pack4(x0 - unpack4(h0)), l1 = pack4(x1 - unpack4(h1));
        const bf16x8 vh = as_bf16x8((u32x4){h0.x, h0.y, h1.x, h1.y}), vl = as_bf16x8((u32x4){l0.x, l0.y, l1.x, l1.y});
#pragma unroll
        for (int i = 0; i < NS; ++i) {
          const bf16_t* kt = s_k + (s + (li >> 2)) * PK + i * 16 + (li & 3) * 4;
          const u32x2 lo = lds_read_tr(kt), hi = lds_read_tr(kt + 4 * PK);
          const bf16x8 kf = as_bf16x8((u32x4){lo.x, lo.y, hi.x, hi.y});
          st[i] = mfma16(kf, vh, st[i]);
          st[i] = mfma16(kf, vl, st[i]);
        }
      }
    }
    __syncthreads();
  }
  if (OUT && SEGMENT) return;
#pragma unroll
  for (int i = 0; i < NS; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) S[(size_t)(i * 16 + g * 4 + r) * a.ep] = st[i][r];
  if (SEGMENT && v0 == 0 && tid == 0) a.seg_decay[(size_t)seg * a.heads + h] = total;
}

// phase 2: seg_state of every segment becomes the state it starts from; the slot gets the state behind the last one
__global__ __launch_bounds__(256) void rec_segments_kernel(RecScanArgs a, int pieces) {
  const int str = blockIdx.z, h = blockIdx.y, p = blockIdx.x * 256 + threadIdx.x;
  if (p >= pieces) return;
  const int s0 = a.str_seg0[str], ns = a.str_nseg[str];
  const size_t per = (size_t)a.np * a.ep, hop = (size_t)a.heads * per;
  float* seg = a.seg_state + ((size_t)s0 * a.heads + h) * per + (size_t)p * 4;
  float* S = reinterpret_cast<float*>(a.kv_base[a.seg_slot[s0]] + a.state_off) + (size_t)h * per + (size_t)p * 4;
  f32x4 cur = {0.f, 0.f, 0.f, 0.f};
  if (!a.seg_fresh[s0]) cur = *reinterpret_cast<const f32x4*>(S);
  f32x4 nxt = *reinterpret_cast<const f32x4*>(seg);
  for (int i = 0; i < ns; ++i) {
    const f32x4 own = nxt;
    if (i + 1 < ns) nxt = *reinterpret_cast<const f32x4*>(seg + (size_t)(i + 1) * hop);
    *reinterpret_cast<f32x4*>(seg + (size_t)i * hop) = cur;
    cur = cur * exp2f(a.seg_decay[(size_t)(s0 + i) * a.heads + h]) + own;
  }
  *reinterpret_cast<f32x4*>(S) = cur;
}

template <int NT, bool OUT, bool SEGMENT>
static void scan_go(const RecScanArgs& a, hipStream_t st) {
  constexpr size_t PK = NT * 64 + 8, lds = (64 * PK + 64 * 72) * 2 + 768 + (OUT ? 3 * 64 * PK * 2 : 0);
  static DeviceOnce once;   // per instantiation
  if (once.first()) (void)hipFuncSetAttribute((const void*)rec_scan_kernel<NT, OUT, SEGMENT>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
  rec_scan_kernel<NT, OUT, SEGMENT><<<dim3(a.n_seg, a.heads * (a.ep / 64)), dim3(256), lds, st>>>(a);
}
template <int NT>
static void scan_all(const RecScanArgs& a, hipStream_t st) {
  if (a.n_seg == a.n_streams) { scan_go<NT, true, false>(a, st); return; }
  scan_go<NT, false, true>(a, st);
  const int pieces = a.np * a.ep / 4;
  rec_segments_kernel<<<dim3((pieces + 255) / 256, a.heads, a.n_streams), dim3(256), 0, st>>>(a, pieces);
  scan_go<NT, true, true>(a, st);
}
int rec_scan(const RecScanArgs& a, hipStream_t st) {
  if (a.n_seg <= 0) return 0;
  if (a.heads < 1 || a.groups < 1 || a.heads % a.groups || a.np < 64 || (a.np & 63) || a.np > 256 || a.ep < 64 || (a.ep & 63) || a.heads * (a.ep / 64) > 65535 ||
      a.n_streams < 1 || a.n_streams > 65535 || a.n_seg < a.n_streams) return LCC_ERR_SHAPE;
  if (!a.q || !a.k || !a.v || !a.rate || !a.y || !a.seg_row0 || !a.seg_rows || !a.seg_slot || !a.seg_fresh || !a.kv_base) return LCC_ERR_ARG;
  if (a.n_seg > a.n_streams && (!a.seg_state || !a.seg_decay || !a.str_seg0 || !a.str_nseg)) return LCC_ERR_ARG;
  switch (a.np / 64) {
    case 1: scan_all<1>(a, st); break;
    case 2: scan_all<2>(a, st); break;
    case 3: scan_all<3>(a, st); break;
    default: scan_all<4>(a, st); break;
  }
  return 0;
}

// ------------------------------------------------------------------------------------------------------------------------------
// Behind the recurrence: gated norm, grid (row, norm group); RING: the inputs the convolution of the stream's next call needs
// ------------------------------------------------------------------------------------------------------------------------------
template <bool RING, int NW, int MAXP>
__global__ __launch_bounds__(NW * 64) void rec_norm_kernel(RecNormArgs a, RecInArgs in) {
  __shared__ float red[NW];
  if (RING && blockIdx.y == 0) conv_ring_row<NW>(in, blockIdx.x);
  rec_norm_row<NW, MAXP>(a, blockIdx.x, blockIdx.y, red);
}
bool rec_norm_ok(const RecNormArgs& a) {
  return a.y && a.part && a.nsplit >= 1 && a.w && a.out && a.heads >= 1 && a.vdim >= 1 && a.vdim <= a.ep && !(a.ep & 3) && a.norm_groups >= 1 && a.norm_groups <= 65535 &&
         (a.heads * a.vdim) % a.norm_groups == 0 && a.ld >= a.heads * a.vdim && !(a.ld & 7) && !(a.ldn & 3) && !(a.gate_col & 3) && a.gate_col >= 0 &&
         a.gate_col + a.heads * a.ep <= a.ldn;
}
int rec_norm(const RecNormArgs& a, hipStream_t st) {
  if (a.rows <= 0) return 0;
  if (!rec_norm_ok(a)) return LCC_ERR_SHAPE;
  if (a.conv && (a.conv->taps < 1 || !a.conv->tok_last || !a.conv->tok_pos || !a.conv->tok_stream || !a.conv->kv_base || a.conv->rows != a.rows)) return LCC_ERR_ARG;
  const dim3 grid(a.rows, a.norm_groups);
  const int gs = a.heads * a.vdim / a.norm_groups;
#define LCC_GO(NW, MAXP)                                                                                \
  do {                                                                                                  \
    if (a.conv) rec_norm_kernel<true, NW, MAXP><<<grid, dim3(NW * 64), 0, st>>>(a, *a.conv);            \
    else rec_norm_kernel<false, NW, MAXP><<<grid, dim3(NW * 64), 0, st>>>(a, RecInArgs());              \
  } while (0)
  if (gs <= 1024) LCC_GO(4, 1);
  else if (a.rows <= 64) LCC_GO(16, 2);                // few rows: latency
  else if (gs <= 2048) LCC_GO(4, 2);
  else if (gs <= 4096) LCC_GO(8, 2);
  else LCC_GO(16, 2);
#undef LCC_GO
  return 0;
}

}  // namespace lcc
