// Grouped-head softmax attention over a paged per-token cache on the matrix cores, with what designs put beside the plain scores, each
// a parameter: a sliding window, a linear distance bias per head, a learned sink per head, a sigmoid gate per head.
//
//     s_ij = (q_i . k_j) * scale - slope_h (i - j)          j visible from i  <=>  0 <= i - j < window  (window <= 0: every j <= i)
//     o_i  = sum_j exp(s_ij) v_j / (exp(sink_h) + sum_j exp(s_ij)) * sigmoid(gate_ih)          (no sink: without the first term)
//
//   vlm_qkv_rownorm_rows    packed projection rows -> (x + bias) RMS-normed over ALL heads of q, and of k, at once, times a weight of that
//                           size; q also times 1 + coef * ln(floor((pos + 1) / every) + 1) -> dense fp32 rows; k into the paged key
//                           cache; v + bias, optionally mixed with the values another layer cached for the same token
//                           ((1 - mix) v + mix v_other), into the paged value cache - one launch
//   vlm_grouped_attn_blocks prompt: 16 query columns = up to 16 consecutive tokens of one sequence; CG heads of one key / value head
//                           share the loaded keys and values
//   vlm_grouped_attn_rows   decode: 16 query columns = up to 16 of the query heads that share a key / value head, one token; `nsplit`
//                           workgroups share the keys of a column group and leave partial results that a second kernel merges
//
// q fp32 [tokens][H][D], values T [pages][64][KH][Dv], output T rows [H * Dv].  Query head h reads key / value head h / (H / KH).
// Keys, by T:
//   fp32: [pages][64][KH][D] fp32; products on v_mfma_f32_16x16x4_f32 (true fp32 products and sums).
//   bf16: every key coordinate as the sum of two bf16 values, hi = bf16(k), lo = bf16(k - hi): [pages][64][KH][2 (hi, lo)][D8], D8 = D
//         rounded up to 8 (the padding stays zero).  Queries are split the same way, scores are q_hi k_hi + q_hi k_lo + q_lo k_hi on
//         v_mfma_f32_16x16x32_bf16 with fp32 sums; the softmax weights enter the product with V as hi + lo as well.
//
// The waves (of all splits) take turns over the key tiles (16 or 32 keys at multiples of that counted from the sequence's first token) and
// work straight from global memory in the operand layout, without LDS traffic for keys or values (see attn_mfma.hpp).  Running maximum
// and sum live in registers, per query; a tile without a visible key leaves them bit for bit as they were.  The waves' partial
// results are merged through LDS at the end, in wave order.
#include "common.hpp"
#include "../../include/vlm_hip.h"
#include "recurrence_finish.hpp"
#include "attn_mfma.hpp"

namespace {

constexpr int PAGE = 64, QC = 16;
constexpr float LOG2E = 1.4426950408889634f;

// ---------------------------------------------------------------------------------------------------------------- projection rows
// grid (tokens, 2): y = 0 queries, y = 1 keys and values
template <typename T>
__global__ __launch_bounds__(256) void qkv_rownorm_kernel(vlm_qkv_rownorm_args p) {
  __shared__ float red[4];
  const long t = blockIdx.x;
  const int tid = threadIdx.x, pos = p.tok_pos[t];
  const bool isq = blockIdx.y == 0;
  const int heads = isq ? p.HQ : p.HK, D = p.D, N = heads * D;
  const T* x = (const T*)p.x + t * p.ldx + (isq ? p.qoff : p.koff);
  const T* b = (const T*)(isq ? p.qbias : p.kbias);
  const T* w = (const T*)(isq ? p.qw : p.kw);
  float ss = 0.f;
  for (int i = tid; i < N; i += 256) {
    const float v = ld_f(x + i) + (b ? ld_f(b + i) : 0.f);
    ss = fmaf(v, v, ss);
  }
  ss = wave_sum(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  float r = 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)N + p.eps);
  if (isq) {
    const float mult = p.temp_every > 0 ? 1.f + p.temp_coef * logf((float)((pos + 1) / p.temp_every) + 1.f) : 1.f;
    float* q = p.q + t * N;
    for (int i = tid; i < N; i += 256) q[i] = (ld_f(x + i) + (b ? ld_f(b + i) : 0.f)) * r * ld_f(w + i) * mult;
    return;
  }
  const long row = (long)p.block_table[(long)p.tok_seq[t] * p.max_pages + pos / PAGE] * PAGE + pos % PAGE;
  if (p.k_split) {
    const int D8 = (D + 7) & ~7;
    bf16_t* kr = (bf16_t*)p.kpool + row * heads * 2 * D8;
    for (int i = tid; i < N; i += 256) {
      const float v = (ld_f(x + i) + (b ? ld_f(b + i) : 0.f)) * r * ld_f(w + i);
      const bf16_t hi = f2bf(v);
      const int h = i / D;
      kr[h * 2 * D8 + (i - h * D)] = hi;
      kr[h * 2 * D8 + D8 + (i - h * D)] = f2bf(v - bf2f(hi));
    }
  } else {
    float* kr = (float*)p.kpool + row * N;
    for (int i = tid; i < N; i += 256) kr[i] = (ld_f(x + i) + (b ? ld_f(b + i) : 0.f)) * r * ld_f(w + i);
  }
  const T* v = (const T*)p.x + t * p.ldx + p.voff;
  const T* vb = (const T*)p.vbias;
  T* vr = (T*)p.vpool + row * p.NV;
  const T* other = p.vother ? (const T*)p.vother + row * p.NV : nullptr;
  for (int i = tid; i < p.NV; i += 256) {
    float a = ld_f(v + i) + (vb ? ld_f(vb + i) : 0.f);
    if (other) a = (1.f - p.mix) * a + p.mix * ld_f(other + i);
    st_f(vr + i, a);
  }
}

// ---------------------------------------------------------------------------------------------------------------- attention
// scores of 16 keys (this lane's operand row: `kr`) against the CG groups of 16 query columns in LDS
template <int CG>
__device__ __forceinline__ void scores16(const float* kr, bool dvec, int D, int DP, const float* qs, int QP, int r16, int g, f32x4_t* s) {
  const float* q = qs + r16 * QP + 4 * g;
#pragma unroll 4
  for (int c = 0; c < DP; c += 16) {
    float4 k = make_float4(0.f, 0.f, 0.f, 0.f);
    const int d = c + 4 * g;
    if (dvec) {
      if (d < D) k = *reinterpret_cast<const float4*>(kr + d);
    } else {
      if (d + 0 < D) k.x = kr[d + 0];
      if (d + 1 < D) k.y = kr[d + 1];
      if (d + 2 < D) k.z = kr[d + 2];
      if (d + 3 < D) k.w = kr[d + 3];
    }
#pragma unroll
    for (int m = 0; m < CG; ++m) {
      const float4 a = *reinterpret_cast<const float4*>(q + m * QC * QP + c);
      s[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(k.x, a.x, s[m], 0, 0, 0);
      s[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(k.y, a.y, s[m], 0, 0, 0);
      s[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(k.z, a.z, s[m], 0, 0, 0);
      s[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(k.w, a.w, s[m], 0, 0, 0);
    }
  }
}

// queries in LDS: [CG][2 (hi, lo)][QC][QPB] bf16; kr: the key's [2][D8] bf16
template <int CG>
__device__ __forceinline__ void scores16(const bf16_t* kr, int D8, const bf16_t* qb, int QPB, int r16, int g, f32x4_t* s) {
  const bf16_t* q = qb + r16 * QPB + 8 * g;
  const int pl = QC * QPB;
#pragma unroll 2
  for (int c = 0; c < D8; c += 32) {
    const int d = c + 8 * g;
    bf8 kh = zero8(), kl = kh;
    if (d < D8) {
      kh = *reinterpret_cast<const bf8*>(kr + d);
      kl = *reinterpret_cast<const bf8*>(kr + D8 + d);
    }
#pragma unroll
    for (int m = 0; m < CG; ++m) {
      const bf8 qh = *reinterpret_cast<const bf8*>(q + 2 * m * pl + c), ql = *reinterpret_cast<const bf8*>(q + (2 * m + 1) * pl + c);
      s[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kl, qh, s[m], 0, 0, 0);
      s[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kh, ql, s[m], 0, 0, 0);
      s[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kh, qh, s[m], 0, 0, 0);
    }
  }
}

template <typename T> __device__ __forceinline__ float head_gate(const vlm_grouped_attn_args& p, long tok, int h) {
  return p.gate ? 1.f / (1.f + expf(-ld_f((const T*)p.gate + tok * p.ldgate + h))) : 1.f;
}

template <typename T, int NB, int CG, int NW>
__global__ __launch_bounds__(NW * 64) void grouped_attn_kernel(vlm_grouped_attn_args p, int decode, int heads_per_block) {
  constexpr bool F32 = sizeof(T) == 4;
  constexpr int U = F32 ? 1 : 2, KTL = 16 * U;           // 16-key groups per tile, keys per tile
  constexpr int OP = NB * 16 + 4;
  extern __shared__ __align__(16) float smem[];
  const int D = p.D, Dv = p.Dv;
  const int DP = (D + 15) & ~15, QP = DP + 4;            // fp32 queries: [CG][QC][QP]
  const int D8 = (D + 7) & ~7, DPB = (D + 31) & ~31, QPB = DPB + 8;   // bf16 queries: [CG][2][QC][QPB]
  float* qs = smem;                                      // queries times scale * log2(e)
  bf16_t* qb = reinterpret_cast<bf16_t*>(smem);
  float* os = smem;                                      // [CG][QC][OP], in the queries' place once every wave is through its keys
  float* ml = smem + max(F32 ? CG * QC * QP : CG * QC * QPB, CG * QC * OP);   // [NW][CG][QC][2]: running maximum and sum of every wave
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, r16 = lane & 15, g = lane >> 4;
  const int R = p.H / p.KH;
  // the workgroup's columns: column c of group m is (token t0 + c, head h0 + m), decoding (token t0, head h0 + c)
  int t0, ncol, h0, kh, nm = CG;                         // (nm: groups that exist)
  if (decode) {
    const int hb = (R + heads_per_block - 1) / heads_per_block;
    t0 = blockIdx.x;
    kh = blockIdx.y / hb;
    const int o = (blockIdx.y % hb) * heads_per_block;
    h0 = kh * R + o;
    ncol = min(heads_per_block, R - o);
  } else {
    const int b = gridDim.y - 1 - blockIdx.y;            // (the blocks of a prompt's end have the most keys: they start first)
    t0 = p.qb_start[b];
    ncol = p.qb_count[b];
    const int hp = (R + CG - 1) / CG, o = (blockIdx.x % hp) * CG;
    kh = blockIdx.x / hp;
    h0 = kh * R + o;
    nm = min(CG, R - o);
  }
  const int* bt = p.block_table + (long)p.tok_seq[t0] * p.max_pages;
  const int pos0 = p.tok_pos[t0], last = decode ? pos0 : pos0 + ncol - 1;
  const int window = p.window;
  const int tiles = last / KTL + 1;
  const int first_tile = window > 0 ? max(0, pos0 - window + 1) / KTL : 0;   // holds the first query's oldest visible key
  const bool split = gridDim.z > 1;
  if (split && first_tile + (int)blockIdx.z * NW >= tiles) {              // no keys for this workgroup: only the marks of an empty part (uniform)
    if (tid < ncol) {
      float* q = p.part + (((long)blockIdx.z * p.H + h0 + tid) * gridDim.x + t0) * (Dv + 2);
      q[Dv] = -INFINITY;
      q[Dv + 1] = 0.f;
    }
    return;
  }
  const float sc = p.scale * LOG2E;
  const int dq = F32 ? DP : DPB;
  for (int i = tid; i < CG * QC * dq; i += NW * 64) {
    const int d = i % dq, c = (i / dq) % QC, m = i / (dq * QC);
    float v = 0.f;
    if (c < ncol && d < D && m < nm) {
      const long tok = decode ? t0 : t0 + c;
      const int h = decode ? h0 + c : h0 + m;
      v = p.q[(tok * p.H + h) * D + d] * sc;
    }
    if constexpr (F32) {
      qs[(m * QC + c) * QP + d] = v;
    } else {
      const bf16_t hi = f2bf(v);
      qb[((m * 2 + 0) * QC + c) * QPB + d] = hi;
      qb[((m * 2 + 1) * QC + c) * QPB + d] = f2bf(v - bf2f(hi));
    }
  }
  __syncthreads();
  const int mypos = r16 < ncol ? (decode ? pos0 : pos0 + r16) : -1;       // (a column that does not exist sees nothing)
  float slope[CG];                                       // of this lane's column, times log2(e)
#pragma unroll
  for (int m = 0; m < CG; ++m) slope[m] = p.slope ? p.slope[decode ? h0 + min(r16, ncol - 1) : h0 + min(m, nm - 1)] * LOG2E : 0.f;
  f32x4_t acc[CG][NB];
#pragma unroll
  for (int m = 0; m < CG; ++m)
#pragma unroll
    for (int b = 0; b < NB; ++b) acc[m][b] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float mrun[CG], lrun[CG];
#pragma unroll
  for (int m = 0; m < CG; ++m) {
    mrun[m] = -INFINITY;
    lrun[m] = 0.f;
  }
  const bool dvec = (D & 3) == 0, vvec = Dv % NB == 0;
  const int vcol = r16 * NB, vhave = Dv - vcol;
  const long krow_sz = F32 ? (long)p.KH * D : (long)p.KH * 2 * D8, vrow_sz = (long)p.KH * Dv;
  const T* kbase = (const T*)p.kpool + kh * (krow_sz / p.KH);
  const T* vbase = (const T*)p.vpool + (long)kh * Dv + vcol;
  const int nw = NW * gridDim.z;
  for (int j = first_tile + blockIdx.z * NW + wave; j < tiles; j += nw) {
    const long prow = (long)bt[j / (PAGE / KTL)] * PAGE + (j % (PAGE / KTL)) * KTL;
    const int lim = last - j * KTL;                                       // place of the last key that exists (may be past the tile)
    f32x4_t s[U][CG];
#pragma unroll
    for (int u = 0; u < U; ++u) {
#pragma unroll
      for (int m = 0; m < CG; ++m) s[u][m] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      const T* kr = kbase + (prow + min(16 * u + r16, lim)) * krow_sz;
      if constexpr (F32) scores16<CG>(kr, dvec, D, DP, qs, QP, r16, g, s[u]);
      else scores16<CG>(kr, D8, qb, QPB, r16, g, s[u]);
    }
    // values of keys 4 g .. 4 g + 3 of every group (independent of the scores: in flight while the softmax runs)
    VRow<T, NB> v[U * 4];
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int r = 0; r < 4; ++r) v[u * 4 + r].load(vbase + (prow + min(16 * u + 4 * g + r, lim)) * vrow_sz, vhave, vvec);
    // a tile that every query of the workgroup sees in full needs no mask
    const int tile_lo = j * KTL, tile_hi = tile_lo + KTL - 1;
    const bool full = tile_hi <= pos0 && (window <= 0 || last - tile_lo < window);
    float pr[CG][U * 4], al[CG];
    bool moved = false;
#pragma unroll
    for (int m = 0; m < CG; ++m) {
      float mx = -INFINITY;
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int dist = mypos - (tile_lo + 16 * u + 4 * g + r);
          const float v0 = fmaf(-slope[m], (float)dist, s[u][m][r]);
          pr[m][u * 4 + r] = full || (dist >= 0 && (window <= 0 || dist < window)) ? v0 : -INFINITY;
        }
#pragma unroll
      for (int i = 0; i < U * 4; ++i) mx = fmaxf(mx, pr[m][i]);
      mx = col4_max(mx);
      const float m_new = fmaxf(mrun[m], mx), ms = m_new == -INFINITY ? 0.f : m_new;
      al[m] = m_new == -INFINITY ? 1.f : __builtin_amdgcn_exp2f(mrun[m] - ms);      // (nothing seen before: exp2(-inf) = 0)
      mrun[m] = m_new;
      float sum = 0.f;
#pragma unroll
      for (int i = 0; i < U * 4; ++i) {
        pr[m][i] = __builtin_amdgcn_exp2f(pr[m][i] - ms);
        sum += pr[m][i];
      }
      lrun[m] = fmaf(lrun[m], al[m], sum);                                // (this lane's keys only; summed over the column at the end)
      moved |= al[m] != 1.f;
    }
    if (__any(moved)) {
#pragma unroll
      for (int m = 0; m < CG; ++m)
#pragma unroll
        for (int b = 0; b < NB; ++b) acc[m][b] *= al[m];
    }
    if constexpr (F32) {
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int b = 0; b < NB; ++b)
#pragma unroll
          for (int m = 0; m < CG; ++m) acc[m][b] = __builtin_amdgcn_mfma_f32_16x16x4f32(v[r].f[b], pr[m][r], acc[m][b], 0, 0, 0);
    } else {
      bf8 ph[CG], pl[CG];                                                 // contraction index 8 g + i: key 16 (i / 4) + 4 g + i % 4
#pragma unroll
      for (int m = 0; m < CG; ++m) split8(pr[m], ph[m], pl[m]);
#pragma unroll
      for (int b = 0; b < NB; ++b) {
        u32x4_t t;
#pragma unroll
        for (int i = 0; i < 4; ++i) t[i] = pair_cols(v[(2 * i) % (U * 4)].w[b / 2], v[(2 * i + 1) % (U * 4)].w[b / 2], b & 1);
        const bf8 vt = __builtin_bit_cast(bf8, t);
#pragma unroll
        for (int m = 0; m < CG; ++m) {
          acc[m][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt, pl[m], acc[m][b], 0, 0, 0);
          acc[m][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt, ph[m], acc[m][b], 0, 0, 0);
        }
      }
    }
  }
  // merge: common maximum per column, every wave's sums scaled to it and added in wave order
#pragma unroll
  for (int m = 0; m < CG; ++m) {
    lrun[m] = col4_sum(lrun[m]);
    if (g == 0) {
      ml[((wave * CG + m) * QC + r16) * 2] = mrun[m];
      ml[((wave * CG + m) * QC + r16) * 2 + 1] = lrun[m];
    }
  }
  __syncthreads();
#pragma unroll
  for (int m = 0; m < CG; ++m) {
    float M = -INFINITY;
    for (int w = 0; w < NW; ++w) M = fmaxf(M, ml[((w * CG + m) * QC + r16) * 2]);
    const float ms = M == -INFINITY ? 0.f : M;
    float l = 0.f;
    for (int w = 0; w < NW; ++w) l = fmaf(ml[((w * CG + m) * QC + r16) * 2 + 1], __builtin_amdgcn_exp2f(ml[((w * CG + m) * QC + r16) * 2] - ms), l);
    const int h = decode ? h0 + min(r16, ncol - 1) : h0 + min(m, nm - 1);
    if (split) {
      if (wave == 0 && g == 0 && r16 < ncol) {           // (split only when decoding: CG = 1)
        float* q = p.part + (((long)blockIdx.z * p.H + h) * gridDim.x + t0) * (Dv + 2);
        q[Dv] = M;
        q[Dv + 1] = l;
      }
    } else if (p.sink) {
      l += __builtin_amdgcn_exp2f(p.sink[h] * LOG2E - ms);
    }
    const float f = __builtin_amdgcn_exp2f(mrun[m] - ms) * (split ? 1.f : (l > 0.f ? 1.f / l : 0.f));
#pragma unroll
    for (int b = 0; b < NB; ++b) acc[m][b] *= f;
  }
  for (int w = 0; w < NW; ++w) {
    if (wave == w) {
#pragma unroll
      for (int m = 0; m < CG; ++m) {
        float* orow = os + (m * QC + r16) * OP;
#pragma unroll
        for (int b = 0; b < NB; ++b)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int c = (4 * g + r) * NB + b;                           // value column of row 4 g + r of block b
            orow[c] = w == 0 ? acc[m][b][r] : orow[c] + acc[m][b][r];
          }
      }
    }
    __syncthreads();
  }
  for (int i = tid; i < nm * ncol * Dv; i += NW * 64) {
    const int d = i % Dv, c = (i / Dv) % ncol, m = i / (Dv * ncol);
    const long tok = decode ? t0 : t0 + c;
    const int h = decode ? h0 + c : h0 + m;
    const float o = os[(m * QC + c) * OP + d];
    if (split) p.part[(((long)blockIdx.z * p.H + h) * gridDim.x + t0) * (Dv + 2) + d] = o;
    else st_f((T*)p.out + tok * p.ldo + (long)h * Dv + d, o * head_gate<T>(p, tok, h));
  }
}

// merge of the splits' partial results: grid (rows, H), 2 waves (wave w: every other 64 value columns from 64 w).
// part: [split][H][rows][Dv sums | maximum | sum]; the splits that had keys come first
template <typename T>
__global__ __launch_bounds__(128) void grouped_attn_merge_kernel(vlm_grouped_attn_args p, int nsplit) {
  const long t = blockIdx.x;
  const int h = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, Dv = p.Dv;
  const long step = (long)p.H * gridDim.x * (Dv + 2);
  const float* q = p.part + ((long)h * gridDim.x + t) * (Dv + 2);
  const float M_mine = lane < nsplit ? q[lane * step + Dv] : -INFINITY, l_mine = lane < nsplit ? q[lane * step + Dv + 1] : 0.f;
  const float M = wave_max(M_mine), ms = M == -INFINITY ? 0.f : M;
  const float f_mine = __builtin_amdgcn_exp2f(M_mine - ms);
  float l = wave_sum(l_mine * f_mine);
  if (p.sink) l += __builtin_amdgcn_exp2f(p.sink[h] * LOG2E - ms);
  const float inv = (l > 0.f ? 1.f / l : 0.f) * head_gate<T>(p, t, h);
  const int n = __popcll(__ballot(M_mine != -INFINITY));
  for (int c0 = 64 * wave; c0 < Dv; c0 += 128) {         // (whole waves: the shuffles below need every lane)
    const int c = min(c0 + lane, Dv - 1);
    float a = 0.f;
    for (int z0 = 0; z0 < n; z0 += 8) {             // eight loads in flight; splits past the last one count for nothing
      float v[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] = q[min(z0 + i, n - 1) * step + c];
#pragma unroll
      for (int i = 0; i < 8; ++i) a = fmaf(__shfl(f_mine, min(z0 + i, 63)) * (z0 + i < n ? 1.f : 0.f), v[i], a);
    }
    if (c0 + lane < Dv) st_f((T*)p.out + t * p.ldo + (long)h * Dv + c, a * inv);
  }
}

size_t lds_bytes(const vlm_grouped_attn_args& a, int NB, int CG, int NW, bool f32) {
  const size_t q = f32 ? (size_t)CG * QC * (((a.D + 15) & ~15) + 4) : (size_t)CG * QC * (((a.D + 31) & ~31) + 8);
  const size_t o = (size_t)CG * QC * (NB * 16 + 4);
  return ((q > o ? q : o) + (size_t)NW * CG * QC * 2) * sizeof(float);
}

template <typename T, int CG, int NW>
int launch(const vlm_grouped_attn_args& a, dim3 grid, int decode, int hpb, hipStream_t st) {
  const int need = (a.Dv + 15) / 16;
  const int NB = need <= 1 ? 1 : need <= 2 ? 2 : need <= 4 ? 4 : need <= 8 ? 8 : 16;
  const size_t lds = lds_bytes(a, NB, CG, NW, sizeof(T) == 4);
  if (need > 16 || lds > 64 * 1024) return VLM_ERR_SHAPE;
#define GO(N) hipLaunchKernelGGL((grouped_attn_kernel<T, N, CG, NW>), grid, dim3(NW * 64), lds, st, a, decode, hpb)
  if (NB == 1) GO(1); else if (NB == 2) GO(2); else if (NB == 4) GO(4); else if (NB == 8) GO(8); else GO(16);
#undef GO
  VLM_CHECK_LAUNCH();
  return VLM_OK;
}

bool bad(const vlm_grouped_attn_args* a) {
  return !a || !a->q || !a->kpool || !a->vpool || !a->tok_seq || !a->tok_pos || !a->block_table || !a->out || a->max_pages <= 0 || a->H <= 0 ||
         a->KH <= 0 || a->H % a->KH || a->D <= 0 || a->Dv <= 0 || a->ldo < (long)a->H * a->Dv || (a->gate && a->ldgate < a->H);
}

}  // namespace

extern "C" int vlm_qkv_rownorm_rows(const vlm_qkv_rownorm_args* a, int rows, int dtype, void* stream) {
  if (!a || !a->x || !a->qw || !a->kw || !a->tok_seq || !a->tok_pos || !a->block_table || !a->q || !a->kpool || !a->vpool || a->HQ <= 0 ||
      a->HK <= 0 || a->D <= 0 || a->NV <= 0 || a->max_pages <= 0 || rows < 0 || a->qoff < 0 || a->koff < 0 || a->voff < 0 ||
      a->ldx < a->qoff + (long)a->HQ * a->D || a->ldx < a->koff + (long)a->HK * a->D || a->ldx < a->voff + (long)a->NV || (dtype && a->k_split))
    return VLM_ERR_ARG;
  if (rows == 0) return VLM_OK;
  if (dtype) hipLaunchKernelGGL(qkv_rownorm_kernel<float>, dim3(rows, 2), dim3(256), 0, (hipStream_t)stream, *a);
  else hipLaunchKernelGGL(qkv_rownorm_kernel<bf16_t>, dim3(rows, 2), dim3(256), 0, (hipStream_t)stream, *a);
  VLM_CHECK_LAUNCH();
  return VLM_OK;
}

extern "C" int vlm_grouped_attn_blocks(const vlm_grouped_attn_args* a, int nblocks, int dtype, void* stream) {
  if (bad(a) || !a->qb_start || !a->qb_count || nblocks < 0) return VLM_ERR_ARG;
  if (a->H > 65535 || nblocks > 65535) return VLM_ERR_SHAPE;
  if (nblocks == 0) return VLM_OK;
  hipStream_t st = (hipStream_t)stream;
  const int R = a->H / a->KH;
  if (R >= 2) {                                          // two heads share the loaded keys and values (an odd one runs alone)
    const int NB = (a->Dv + 15) / 16 <= 8 ? 8 : 16;
    if (lds_bytes(*a, NB, 2, 4, dtype != 0) <= 64 * 1024) {
      const dim3 grid(a->KH * ((R + 1) / 2), nblocks);
      return dtype ? launch<float, 2, 4>(*a, grid, 0, 16, st) : launch<bf16_t, 2, 4>(*a, grid, 0, 16, st);
    }
  }
  const dim3 grid(a->H, nblocks);
  return dtype ? launch<float, 1, 4>(*a, grid, 0, 16, st) : launch<bf16_t, 1, 4>(*a, grid, 0, 16, st);
}

extern "C" int vlm_grouped_attn_rows(const vlm_grouped_attn_args* a, int rows, int dtype, void* stream) {
  if (bad(a) || rows < 0 || a->nsplit < 0 || a->nsplit > 64 || (a->nsplit > 1 && !a->part)) return VLM_ERR_ARG;
  const int R = a->H / a->KH, hpb = R < 16 ? R : 16;
  const long gy = (long)a->KH * ((R + hpb - 1) / hpb);
  if (gy > 65535 || a->H > 65535) return VLM_ERR_SHAPE;
  if (rows == 0) return VLM_OK;
  const int nsplit = a->nsplit > 1 ? a->nsplit : 1;
  const dim3 grid(rows, (unsigned)gy, nsplit);
  hipStream_t st = (hipStream_t)stream;
  const int rc = dtype ? launch<float, 1, 4>(*a, grid, 1, hpb, st) : launch<bf16_t, 1, 4>(*a, grid, 1, hpb, st);
  if (rc || nsplit == 1) return rc;
  if (dtype) hipLaunchKernelGGL(grouped_attn_merge_kernel<float>, dim3(rows, a->H), dim3(128), 0, st, *a, nsplit);
  else hipLaunchKernelGGL(grouped_attn_merge_kernel<bf16_t>, dim3(rows, a->H), dim3(128), 0, st, *a, nsplit);
  VLM_CHECK_LAUNCH();
  return VLM_OK;
}
