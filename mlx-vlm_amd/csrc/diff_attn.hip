// Differential attention over a paged per-token cache: every head has TWO softmax maps over the same values, and its output is
// their difference:
//
//     s^m_ij = (q^m_i . k^m_j) * scale                              m = 1, 2
//     j visible from i  <=>  j <= i and (window <= 0 or i - j < window or j < keep)      (a sliding window that keeps the first
//                                                                                         `keep` tokens of the sequence in view)
//     a^m_i = sum_j softmax_j(s^m_ij) v_j
//     d_i   = a^1_i - lambda a^2_i         o_i = d_i / sqrt(mean(d_i^2) + eps) * mult       (mean over the head's value columns)
//
// q fp32 [tokens][H][2][D], values T [pages][64][KH][Dv], output T rows [H * Dv].  Query head h reads key / value head h / (H / KH).
// Keys, by T:
//   fp32: [pages][64][KH][2][D] fp32; products on v_mfma_f32_16x16x4_f32 (true fp32 products and sums).
//   bf16: every key coordinate as the sum of two bf16 values, hi = bf16(k), lo = bf16(k - hi): [pages][64][KH][2][2 (hi, lo)][D8], D8 =
//         D rounded up to 8 (the padding stays zero) - the bytes of an fp32 key and 16 bits of its mantissa.  Queries are split the same
//         way, scores are q_hi k_hi + q_hi k_lo + q_lo k_hi on v_mfma_f32_16x16x32_bf16 with fp32 sums; the softmax weights enter
//         the product with V as hi + lo as well, so nothing of a score or a weight is rounded to 8 bits.
//
// One kernel, two forms of a workgroup's 16 query COLUMNS:
//   vlm_diff_attn_blocks  prompt: up to 16 consecutive tokens of one sequence, one head
//   vlm_diff_attn_rows    decode: one token, up to 16 of the query heads that share a key / value head: the head group's keys and
//                         values are read once; `nsplit` workgroups share the keys of a column group and leave partial results
//                         that a second kernel merges
// The waves (of all splits) take turns over the key tiles (16 or 32 keys at multiples of that counted from the sequence's first
// token) and work straight from global memory in the operand layout, without LDS traffic for keys or values: S^T = K Q^T leaves the
// scores of a query in one lane column, with keys 4 g + r of a 16-key group in register r of lane group g - which is the operand
// layout of P^T in O^T += V^T P^T when the contraction runs over the keys in that order.  Lane (r16, g) therefore loads 16 bytes
// of key r16 and NB consecutive value columns of keys 4 g .. 4 g + 3.  Running maximum and sum live in registers, per query; a tile
// without a visible key leaves them bit for bit as they were.  The waves' partial results are merged through LDS at the end, in wave
// order, and the difference, its norm and the store follow.
#include "common.hpp"
#include "../../include/vlm_hip.h"
#include "recurrence_finish.hpp"
#include "attn_mfma.hpp"

namespace {

constexpr int PAGE = 64, QC = 16;

// scores of 16 keys (this lane's operand row: `kr`) against the 16 query columns in LDS, both maps
__device__ __forceinline__ void scores16(const float* kr, bool dvec, int D, int DP, const float* qs, int QP, int r16, int g, f32x4_t& s0, f32x4_t& s1) {
  const float* q0 = qs + r16 * QP + 4 * g;
  const float* q1 = q0 + QC * QP;
#pragma unroll 4
  for (int c = 0; c < DP; c += 16) {
    float4 k0 = make_float4(0.f, 0.f, 0.f, 0.f), k1 = k0;
    const int d = c + 4 * g;
    if (dvec) {
      if (d < D) {
        k0 = *reinterpret_cast<const float4*>(kr + d);
        k1 = *reinterpret_cast<const float4*>(kr + D + d);
      }
    } else {
      if (d + 0 < D) { k0.x = kr[d + 0]; k1.x = kr[D + d + 0]; }
      if (d + 1 < D) { k0.y = kr[d + 1]; k1.y = kr[D + d + 1]; }
      if (d + 2 < D) { k0.z = kr[d + 2]; k1.z = kr[D + d + 2]; }
      if (d + 3 < D) { k0.w = kr[d + 3]; k1.w = kr[D + d + 3]; }
    }
    const float4 a0 = *reinterpret_cast<const float4*>(q0 + c), a1 = *reinterpret_cast<const float4*>(q1 + c);
    s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(k0.x, a0.x, s0, 0, 0, 0);
    s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(k1.x, a1.x, s1, 0, 0, 0);
    s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(k0.y, a0.y, s0, 0, 0, 0);
    s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(k1.y, a1.y, s1, 0, 0, 0);
    s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(k0.z, a0.z, s0, 0, 0, 0);
    s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(k1.z, a1.z, s1, 0, 0, 0);
    s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(k0.w, a0.w, s0, 0, 0, 0);
    s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(k1.w, a1.w, s1, 0, 0, 0);
  }
}

// queries in LDS: [2 maps][2 (hi, lo)][QC][QPB] bf16; kr: the key's [2][2][D8] bf16
__device__ __forceinline__ void scores16(const bf16_t* kr, int D8, const bf16_t* qb, int QPB, int r16, int g, f32x4_t& s0, f32x4_t& s1) {
  const bf16_t* q = qb + r16 * QPB + 8 * g;
  const int pl = QC * QPB;
#pragma unroll 2
  for (int c = 0; c < D8; c += 32) {
    const int d = c + 8 * g;
    bf8 k0h = zero8(), k0l = k0h, k1h = k0h, k1l = k0h;
    if (d < D8) {
      k0h = *reinterpret_cast<const bf8*>(kr + d);
      k0l = *reinterpret_cast<const bf8*>(kr + D8 + d);
      k1h = *reinterpret_cast<const bf8*>(kr + 2 * D8 + d);
      k1l = *reinterpret_cast<const bf8*>(kr + 3 * D8 + d);
    }
    const bf8 q0h = *reinterpret_cast<const bf8*>(q + c), q0l = *reinterpret_cast<const bf8*>(q + pl + c);
    const bf8 q1h = *reinterpret_cast<const bf8*>(q + 2 * pl + c), q1l = *reinterpret_cast<const bf8*>(q + 3 * pl + c);
    s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k0l, q0h, s0, 0, 0, 0);
    s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k1l, q1h, s1, 0, 0, 0);
    s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k0h, q0l, s0, 0, 0, 0);
    s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k1h, q1l, s1, 0, 0, 0);
    s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k0h, q0h, s0, 0, 0, 0);
    s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k1h, q1h, s1, 0, 0, 0);
  }
}

// the shared tail: d = o1 / l1 - lambda o2 / l2 over one head's value columns by 16 neighbouring lanes (l16: the lane's place)
template <typename T, typename F1, typename F2>
__device__ __forceinline__ void difference_store(F1 o1, F2 o2, int Dv, float lambda, float eps, float mult, int l16, bool live, T* out) {
  float ss = 0.f;
  for (int i = l16; i < Dv; i += 16) {
    const float d = o1(i) - lambda * o2(i);
    ss = fmaf(d, d, ss);
  }
#pragma unroll
  for (int o = 8; o > 0; o >>= 1) ss += __shfl_xor(ss, o);
  if (!live) return;
  const float r = mult / sqrtf(ss / (float)Dv + eps);
  for (int i = l16; i < Dv; i += 16) st_f(out + i, (o1(i) - lambda * o2(i)) * r);
}

template <typename T, int NB, int NW>
__global__ __launch_bounds__(NW * 64) void diff_attn_kernel(vlm_diff_attn_args p, int decode, int heads_per_block) {
  constexpr bool F32 = sizeof(T) == 4;
  constexpr int U = F32 ? 1 : 2, KTL = 16 * U;           // 16-key groups per tile, keys per tile
  constexpr int OP = NB * 16 + 4;
  extern __shared__ __align__(16) float smem[];
  const int D = p.D, Dv = p.Dv;
  const int DP = (D + 15) & ~15, QP = DP + 4;            // fp32 queries: [2][QC][QP]
  const int D8 = (D + 7) & ~7, DPB = (D + 31) & ~31, QPB = DPB + 8;   // bf16 queries: [2][2][QC][QPB]
  float* qs = smem;                                      // queries times scale * log2(e)
  bf16_t* qb = reinterpret_cast<bf16_t*>(smem);
  float* os = smem;                                      // [2][QC][OP], in the queries' place once every wave is through its keys
  float* ml = smem + max(F32 ? 2 * QC * QP : 2 * QC * QPB, 2 * QC * OP);   // [NW][2][QC][2]: running maximum and sum of every wave
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, r16 = lane & 15, g = lane >> 4;
  const int R = p.H / p.KH;
  // the workgroup's columns
  int t0, ncol, h0, kh;                                  // first token, number of columns, first head
  if (decode) {
    const int hb = (R + heads_per_block - 1) / heads_per_block;
    t0 = blockIdx.x;
    kh = blockIdx.y / hb;
    const int o = (blockIdx.y % hb) * heads_per_block;
    h0 = kh * R + o;
    ncol = min(heads_per_block, R - o);
  } else {
    t0 = p.qb_start[blockIdx.x];
    ncol = p.qb_count[blockIdx.x];
    h0 = blockIdx.y;
    kh = h0 / R;
  }
  const int* bt = p.block_table + (long)p.tok_seq[t0] * p.max_pages;
  const int pos0 = p.tok_pos[t0], last = decode ? pos0 : pos0 + ncol - 1;
  const float sc = p.scale * 1.4426950408889634f;
  const int dq = F32 ? DP : DPB;
  for (int i = tid; i < 2 * QC * dq; i += NW * 64) {
    const int d = i % dq, c = (i / dq) % QC, m = i / (dq * QC);
    float v = 0.f;
    if (c < ncol && d < D) {
      const long tok = decode ? t0 : t0 + c;
      const int h = decode ? h0 + c : h0;
      v = p.q[((tok * p.H + h) * 2 + m) * D + d] * sc;
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
  const int window = p.window, keep = p.keep;
  f32x4_t acc[2][NB];
#pragma unroll
  for (int m = 0; m < 2; ++m)
#pragma unroll
    for (int b = 0; b < NB; ++b) acc[m][b] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float mrun[2] = {-INFINITY, -INFINITY}, lrun[2] = {0.f, 0.f};
  const int tiles = last / KTL + 1;
  int kept_tiles = 0, first_tile = 0;
  if (window > 0) {
    first_tile = max(0, pos0 - window + 1) / KTL;                         // the first query's oldest key inside the window
    kept_tiles = min((min(keep, last + 1) + KTL - 1) / KTL, first_tile);
  }
  const bool dvec = (D & 3) == 0, vvec = Dv % NB == 0;
  const int vcol = r16 * NB, vhave = Dv - vcol;
  const long krow_sz = F32 ? (long)p.KH * 2 * D : (long)p.KH * 4 * D8, vrow_sz = (long)p.KH * Dv;
  const T* kbase = (const T*)p.kpool + kh * (krow_sz / p.KH);
  const T* vbase = (const T*)p.vpool + (long)kh * Dv + vcol;
  // this wave's tiles: j = its number (mod the number of waves of all splits), those below kept_tiles, then those from first_tile on
  const int nw = NW * gridDim.z;
  int j = blockIdx.z * NW + wave;
  if (j >= kept_tiles && j < first_tile) j += (first_tile - j + nw - 1) / nw * nw;
  while (j < tiles) {
    const long prow = (long)bt[j / (PAGE / KTL)] * PAGE + (j % (PAGE / KTL)) * KTL;
    const int lim = last - j * KTL;                                       // place of the last key that exists (may be past the tile)
    f32x4_t s[U][2];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      s[u][0] = s[u][1] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      const T* kr = kbase + (prow + min(16 * u + r16, lim)) * krow_sz;
      if constexpr (F32) scores16(kr, dvec, D, DP, qs, QP, r16, g, s[u][0], s[u][1]);
      else scores16(kr, D8, qb, QPB, r16, g, s[u][0], s[u][1]);
    }
    // values of keys 4 g .. 4 g + 3 of every group (independent of the scores: in flight while the softmax runs)
    VRow<T, NB> v[U * 4];
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int r = 0; r < 4; ++r) v[u * 4 + r].load(vbase + (prow + min(16 * u + 4 * g + r, lim)) * vrow_sz, vhave, vvec);
    // a tile that every query of the workgroup sees in full needs no mask
    const int tile_lo = j * KTL, tile_hi = tile_lo + KTL - 1;
    const bool full = tile_hi <= pos0 && (window <= 0 || last - tile_lo < window || tile_hi < keep);
    // softmax update of this lane's query column, per map
    float pr[2][U * 4], al[2];
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      float mx = -INFINITY;
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int r = 0; r < 4; ++r) pr[m][u * 4 + r] = s[u][m][r];
      if (!full) {
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int key = tile_lo + 16 * u + 4 * g + r, dist = mypos - key;
            const bool seen = dist >= 0 && (window <= 0 || dist < window || key < keep);
            pr[m][u * 4 + r] = seen ? pr[m][u * 4 + r] : -INFINITY;
          }
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
    }
    if (__any(al[0] != 1.f || al[1] != 1.f)) {
#pragma unroll
      for (int m = 0; m < 2; ++m)
#pragma unroll
        for (int b = 0; b < NB; ++b) acc[m][b] *= al[m];
    }
    if constexpr (F32) {
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int b = 0; b < NB; ++b) {
          acc[0][b] = __builtin_amdgcn_mfma_f32_16x16x4f32(v[r].f[b], pr[0][r], acc[0][b], 0, 0, 0);
          acc[1][b] = __builtin_amdgcn_mfma_f32_16x16x4f32(v[r].f[b], pr[1][r], acc[1][b], 0, 0, 0);
        }
    } else {
      bf8 ph[2], pl[2];                                                   // contraction index 8 g + i: key 16 (i / 4) + 4 g + i % 4
#pragma unroll
      for (int m = 0; m < 2; ++m) {
        u32x4_t h, l;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float a = pr[m][2 * i], b = pr[m][2 * i + 1];
          const unsigned hw = pack_bf2(a, b);
          h[i] = hw;
          l[i] = pack_bf2(a - bf_lo(hw), b - bf_hi(hw));
        }
        ph[m] = __builtin_bit_cast(bf8, h);
        pl[m] = __builtin_bit_cast(bf8, l);
      }
#pragma unroll
      for (int b = 0; b < NB; ++b) {
        u32x4_t t;
#pragma unroll
        for (int i = 0; i < 4; ++i) t[i] = pair_cols(v[(2 * i) % (U * 4)].w[b / 2], v[(2 * i + 1) % (U * 4)].w[b / 2], b & 1);
        const bf8 vt = __builtin_bit_cast(bf8, t);
        acc[0][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt, pl[0], acc[0][b], 0, 0, 0);
        acc[1][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt, pl[1], acc[1][b], 0, 0, 0);
        acc[0][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt, ph[0], acc[0][b], 0, 0, 0);
        acc[1][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt, ph[1], acc[1][b], 0, 0, 0);
      }
    }
    j += nw;
    if (j >= kept_tiles && j < first_tile) j += (first_tile - j + nw - 1) / nw * nw;
  }
  // merge: common maximum per column, every wave's sums scaled to it and added in wave order
#pragma unroll
  for (int m = 0; m < 2; ++m) {
    lrun[m] = col4_sum(lrun[m]);
    if (g == 0) {
      ml[((wave * 2 + m) * QC + r16) * 2] = mrun[m];
      ml[((wave * 2 + m) * QC + r16) * 2 + 1] = lrun[m];
    }
  }
  __syncthreads();
  const bool split = gridDim.z > 1;
#pragma unroll
  for (int m = 0; m < 2; ++m) {
    float M = -INFINITY;
    for (int w = 0; w < NW; ++w) M = fmaxf(M, ml[((w * 2 + m) * QC + r16) * 2]);
    const float ms = M == -INFINITY ? 0.f : M;
    float l = 0.f;
    for (int w = 0; w < NW; ++w) l = fmaf(ml[((w * 2 + m) * QC + r16) * 2 + 1], __builtin_amdgcn_exp2f(ml[((w * 2 + m) * QC + r16) * 2] - ms), l);
    const float f = __builtin_amdgcn_exp2f(mrun[m] - ms) * (split ? 1.f : (l > 0.f ? 1.f / l : 0.f));
#pragma unroll
    for (int b = 0; b < NB; ++b) acc[m][b] *= f;
    if (split && wave == 0 && g == 0 && r16 < ncol) {
      float* q = p.part + (((long)blockIdx.z * p.H + h0 + r16) * gridDim.x + t0) * 2 * (Dv + 2) + m * (Dv + 2);
      q[Dv] = M;
      q[Dv + 1] = l;
    }
  }
  for (int w = 0; w < NW; ++w) {
    if (wave == w) {
#pragma unroll
      for (int m = 0; m < 2; ++m) {
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
  if (split) {
    for (int i = tid; i < ncol * 2 * Dv; i += NW * 64) {
      const int c = i / (2 * Dv), m = (i / Dv) & 1, d = i % Dv;
      p.part[(((long)blockIdx.z * p.H + h0 + c) * gridDim.x + t0) * 2 * (Dv + 2) + m * (Dv + 2) + d] = os[(m * QC + c) * OP + d];
    }
    return;
  }
  // difference, norm over the head's columns, store: 16 lanes per column of the first 4 waves
  if (tid < 256) {
    const int c = tid >> 4, l16 = tid & 15;
    const float* o1 = os + c * OP;
    const float* o2 = o1 + QC * OP;
    const long tok = decode ? t0 : t0 + c;
    const int h = decode ? h0 + c : h0;
    difference_store<T>([&](int i) { return o1[i]; }, [&](int i) { return o2[i]; }, Dv, p.lambda, p.eps, p.mult, l16, c < ncol,
                        (T*)p.out + tok * p.ldo + (long)h * Dv);
  }
}

// merge of the splits' partial results: grid (rows, H), 4 waves (wave w: map w & 1, every other 64 value columns from 64 (w >> 1)).
// part: [split][H][rows][2 maps][Dv sums | maximum | sum]
template <typename T>
__global__ __launch_bounds__(256) void diff_attn_merge_kernel(vlm_diff_attn_args p, int nsplit) {
  extern __shared__ float sm[];                          // [2][Dv]
  const long t = blockIdx.x;
  const int h = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, m = wave & 1, Dv = p.Dv;
  const long step = (long)p.H * gridDim.x * 2 * (Dv + 2);
  const float* q = p.part + (((long)h * gridDim.x + t) * 2 + m) * (Dv + 2);
  const float M_mine = lane < nsplit ? q[lane * step + Dv] : -INFINITY, l_mine = lane < nsplit ? q[lane * step + Dv + 1] : 0.f;
  const float M = wave_max(M_mine);
  const float f_mine = M == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(M_mine - M);
  const float l = wave_sum(l_mine * f_mine), inv = l > 0.f ? 1.f / l : 0.f;
  for (int c0 = 64 * (wave >> 1); c0 < Dv; c0 += 128) {  // (whole waves: the shuffles below need every lane)
    const int c = min(c0 + lane, Dv - 1);
    float a = 0.f;
    for (int z0 = 0; z0 < nsplit; z0 += 8) {             // eight loads in flight; splits past the last one count for nothing
      float v[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] = q[min(z0 + i, nsplit - 1) * step + c];
#pragma unroll
      for (int i = 0; i < 8; ++i) a = fmaf(__shfl(f_mine, min(z0 + i, 63)) * (z0 + i < nsplit ? 1.f : 0.f), v[i], a);
    }
    if (c0 + lane < Dv) sm[m * Dv + c] = a * inv;
  }
  __syncthreads();
  if (wave) return;
  const float* o1 = sm;
  const float* o2 = sm + Dv;
  difference_store<T>([&](int i) { return o1[i]; }, [&](int i) { return o2[i]; }, Dv, p.lambda, p.eps, p.mult, lane & 15, lane < 16,
                      (T*)p.out + t * p.ldo + (long)h * Dv);
}

size_t lds_bytes(const vlm_diff_attn_args& a, int NB, int NW, bool f32) {
  const size_t q = f32 ? (size_t)2 * QC * (((a.D + 15) & ~15) + 4) : (size_t)2 * QC * (((a.D + 31) & ~31) + 8);
  const size_t o = (size_t)2 * QC * (NB * 16 + 4);
  return ((q > o ? q : o) + (size_t)NW * 2 * QC * 2) * sizeof(float);
}

template <typename T, int NW>
int launch(const vlm_diff_attn_args& a, dim3 grid, int decode, int hpb, hipStream_t st) {
  const int need = (a.Dv + 15) / 16;
  const int NB = need <= 1 ? 1 : need <= 2 ? 2 : need <= 4 ? 4 : need <= 8 ? 8 : 16;
  const size_t lds = lds_bytes(a, NB, NW, sizeof(T) == 4);
  if (need > 16 || lds > 64 * 1024) return VLM_ERR_SHAPE;
#define GO(N) hipLaunchKernelGGL((diff_attn_kernel<T, N, NW>), grid, dim3(NW * 64), lds, st, a, decode, hpb)
  if (NB == 1) GO(1); else if (NB == 2) GO(2); else if (NB == 4) GO(4); else if (NB == 8) GO(8); else GO(16);
#undef GO
  VLM_CHECK_LAUNCH();
  return VLM_OK;
}

bool bad(const vlm_diff_attn_args* a) {
  return !a || !a->q || !a->kpool || !a->vpool || !a->tok_seq || !a->tok_pos || !a->block_table || !a->out || a->max_pages <= 0 || a->H <= 0 ||
         a->KH <= 0 || a->H % a->KH || a->D <= 0 || a->Dv <= 0 || a->keep < 0 || a->ldo < (long)a->H * a->Dv;
}

}  // namespace

extern "C" int vlm_diff_attn_blocks(const vlm_diff_attn_args* a, int nblocks, int dtype, void* stream) {
  if (bad(a) || !a->qb_start || !a->qb_count || nblocks < 0) return VLM_ERR_ARG;
  if (a->H > 65535) return VLM_ERR_SHAPE;
  if (nblocks == 0) return VLM_OK;
  const dim3 grid(nblocks, a->H);
  return dtype ? launch<float, 4>(*a, grid, 0, 16, (hipStream_t)stream) : launch<bf16_t, 4>(*a, grid, 0, 16, (hipStream_t)stream);
}

extern "C" int vlm_diff_attn_rows(const vlm_diff_attn_args* a, int rows, int dtype, void* stream) {
  if (bad(a) || rows < 0 || a->nsplit < 0 || a->nsplit > 64 || (a->nsplit > 1 && !a->part)) return VLM_ERR_ARG;
  const int R = a->H / a->KH, hpb = R < 16 ? R : 16;
  const long gy = (long)a->KH * ((R + hpb - 1) / hpb);
  if (gy > 65535 || a->H > 65535) return VLM_ERR_SHAPE;
  if (rows == 0) return VLM_OK;
  const int nsplit = a->nsplit > 1 ? a->nsplit : 1;
  const dim3 grid(rows, (unsigned)gy, nsplit);
  hipStream_t st = (hipStream_t)stream;
  const int rc = dtype ? launch<float, 4>(*a, grid, 1, hpb, st) : launch<bf16_t, 4>(*a, grid, 1, hpb, st);
  if (rc || nsplit == 1) return rc;
  const size_t lds = (size_t)2 * a->Dv * sizeof(float);
  if (dtype) hipLaunchKernelGGL(diff_attn_merge_kernel<float>, dim3(rows, a->H), dim3(256), lds, st, *a, nsplit);
  else hipLaunchKernelGGL(diff_attn_merge_kernel<bf16_t>, dim3(rows, a->H), dim3(256), lds, st, *a, nsplit);
  VLM_CHECK_LAUNCH();
  return VLM_OK;
}
