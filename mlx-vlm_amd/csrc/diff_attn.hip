// Differential attention over a paged per-token cache: every head has TWO softmax maps over the same values, and its output is
// their difference:
//
//     s^m_ij = (q^m_i . k^m_j) * scale                              m = 1, 2
//     j visible from i  <=>  j <= i and (window <= 0 or i - j < window or j < keep)      (a sliding window that keeps the first
//                                                                                         `keep` tokens of the sequence in view)
//     a^m_i = sum_j softmax_j(s^m_ij) v_j
//     d_i   = a^1_i - lambda a^2_i         o_i = d_i / sqrt(mean(d_i^2) + eps) * mult       (mean over the head's value columns)
//
// q fp32 [tokens][H][2][D] (scores are fp32 sums of fp32 products), keys fp32 [pages][64][KH][2][D], values T [pages][64][KH][Dv],
// output T rows [H * Dv].  Query head h reads key / value head h / (H / KH).
//
// One kernel, two forms of a workgroup's 16 query COLUMNS:
//   vlm_diff_attn_blocks  prompt: up to 16 consecutive tokens of one sequence, one head
//   vlm_diff_attn_rows    decode: one token, up to 16 of the query heads that share a key / value head: the head group's keys and
//                         values are read once
// The waves of a workgroup split the key tiles (16 keys at multiples of 16 counted from the sequence's first token, tile j to wave
// j mod NW whatever the step looks like) and run on the fp32 matrix cores (v_mfma_f32_16x16x4_f32: true fp32 products and sums) with
// no LDS traffic for keys or values: S^T = K Q^T leaves the scores of a query in one lane column, with keys 4 g + r in register r
// of lane group g - which is exactly the operand layout of P^T in O^T += V^T P^T when step r contracts the keys 4 g + r.  Lane
// (r16, g) therefore loads 16 bytes of key r16 (dimensions 16 c + 4 g ..) and NB consecutive value columns of keys 4 g .. 4 g + 3.
// Running maximum and sum live in registers, per query; a tile without a visible key leaves them bit for bit as they were.  The
// waves' partial results are merged through LDS at the end, in wave order, and the difference, its norm and the store follow.
#include "common.hpp"
#include "../../include/vlm_hip.h"
#include "recurrence_finish.hpp"

namespace {

constexpr int PAGE = 64, QC = 16, KT = 16;

// NB consecutive value columns; `have`: how many of them exist (<= 0: none)
template <int NB> __device__ __forceinline__ void load_cols(const float* p, int have, bool vec, float* f) {
  if (vec && NB >= 4) {
    if (have > 0) {
#pragma unroll
      for (int i = 0; i < NB / 4; ++i) {
        const float4 a = reinterpret_cast<const float4*>(p)[i];
        f[4 * i] = a.x; f[4 * i + 1] = a.y; f[4 * i + 2] = a.z; f[4 * i + 3] = a.w;
      }
    } else {
#pragma unroll
      for (int i = 0; i < NB; ++i) f[i] = 0.f;
    }
  } else {
#pragma unroll
    for (int i = 0; i < NB; ++i) f[i] = i < have ? p[i] : 0.f;
  }
}
template <int NB> __device__ __forceinline__ void load_cols(const bf16_t* p, int have, bool vec, float* f) {
  if (vec && NB >= 8) {
    if (have > 0) {
#pragma unroll
      for (int i = 0; i < NB / 8; ++i) {
        const uint4 a = reinterpret_cast<const uint4*>(p)[i];
        float* o = f + 8 * i;
        o[0] = bf_lo(a.x); o[1] = bf_hi(a.x); o[2] = bf_lo(a.y); o[3] = bf_hi(a.y);
        o[4] = bf_lo(a.z); o[5] = bf_hi(a.z); o[6] = bf_lo(a.w); o[7] = bf_hi(a.w);
      }
    } else {
#pragma unroll
      for (int i = 0; i < NB; ++i) f[i] = 0.f;
    }
  } else if (vec && NB == 4) {
    uint2 a = make_uint2(0u, 0u);
    if (have > 0) a = *reinterpret_cast<const uint2*>(p);
    f[0] = bf_lo(a.x); f[1 % NB] = bf_hi(a.x); f[2 % NB] = bf_lo(a.y); f[3 % NB] = bf_hi(a.y);
  } else {
#pragma unroll
    for (int i = 0; i < NB; ++i) f[i] = i < have ? bf2f(p[i]) : 0.f;
  }
}

template <typename T, int NB, int NW>
__global__ __launch_bounds__(NW * 64) void diff_attn_kernel(vlm_diff_attn_args p, int decode, int heads_per_block) {
  extern __shared__ __align__(16) float smem[];
  const int D = p.D, Dv = p.Dv, DP = (D + 15) & ~15, QP = DP + 4;
  float* qs = smem;                       // [2][QC][QP], queries times scale * log2(e)
  float* ml = qs + 2 * QC * QP;           // [NW][2][QC][2]: running maximum and sum of every wave
  float* os = ml + NW * 2 * QC * 2;       // [2][QC][NB * 16 + 4]
  constexpr int OP = NB * 16 + 4;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, r16 = lane & 15, g = lane >> 4;
  const int R = p.H / p.KH;
  // the workgroup's columns
  int t0, ncol, h0, kh;                   // first token, number of columns, first head
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
  for (int i = tid; i < 2 * QC * DP; i += NW * 64) {
    const int d = i % DP, c = (i / DP) % QC, m = i / (DP * QC);
    float v = 0.f;
    if (c < ncol && d < D) {
      const long tok = decode ? t0 : t0 + c;
      const int h = decode ? h0 + c : h0;
      v = p.q[((tok * p.H + h) * 2 + m) * D + d] * sc;
    }
    qs[(m * QC + c) * QP + d] = v;
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
  const int tiles = last / KT + 1;
  int kept_tiles = 0, first_tile = 0;
  if (window > 0) {
    first_tile = max(0, pos0 - window + 1) / KT;                          // the first query's oldest key inside the window
    kept_tiles = min((min(keep, last + 1) + KT - 1) / KT, first_tile);
  }
  const bool dvec = (D & 3) == 0, vvec = Dv % NB == 0;
  const int vcol = r16 * NB, vhave = Dv - vcol;
  const long krow_sz = (long)p.KH * 2 * D, vrow_sz = (long)p.KH * Dv;
  const float* kbase = p.kpool + (long)kh * 2 * D;
  const T* vbase = (const T*)p.vpool + (long)kh * Dv + vcol;
  // this wave's tiles: j = wave (mod NW), those below kept_tiles, then those from first_tile on
  int j = wave;
  if (j >= kept_tiles && j < first_tile) j += (first_tile - j + NW - 1) / NW * NW;
  while (j < tiles) {
    const long prow = (long)bt[j / (PAGE / KT)] * PAGE + (j % (PAGE / KT)) * KT;
    const int lim = last - j * KT;                                        // place of the last key that exists (may be >= 16)
    // scores
    f32x4_t s[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
    {
      const float* kr = kbase + (prow + min(r16, lim)) * krow_sz;
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
        s[0] = __builtin_amdgcn_mfma_f32_16x16x4f32(k0.x, a0.x, s[0], 0, 0, 0);
        s[1] = __builtin_amdgcn_mfma_f32_16x16x4f32(k1.x, a1.x, s[1], 0, 0, 0);
        s[0] = __builtin_amdgcn_mfma_f32_16x16x4f32(k0.y, a0.y, s[0], 0, 0, 0);
        s[1] = __builtin_amdgcn_mfma_f32_16x16x4f32(k1.y, a1.y, s[1], 0, 0, 0);
        s[0] = __builtin_amdgcn_mfma_f32_16x16x4f32(k0.z, a0.z, s[0], 0, 0, 0);
        s[1] = __builtin_amdgcn_mfma_f32_16x16x4f32(k1.z, a1.z, s[1], 0, 0, 0);
        s[0] = __builtin_amdgcn_mfma_f32_16x16x4f32(k0.w, a0.w, s[0], 0, 0, 0);
        s[1] = __builtin_amdgcn_mfma_f32_16x16x4f32(k1.w, a1.w, s[1], 0, 0, 0);
      }
    }
    // values of keys 4 g .. 4 g + 3 (independent of the scores: in flight while the softmax runs)
    float v[4][NB];
#pragma unroll
    for (int r = 0; r < 4; ++r) load_cols<NB>(vbase + (prow + min(4 * g + r, lim)) * vrow_sz, vhave, vvec, v[r]);
    // softmax update of this lane's query column, per map
    float pr[2][4], al[2];
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      float mx = -INFINITY;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = j * KT + 4 * g + r, dist = mypos - key;
        const bool seen = dist >= 0 && (window <= 0 || dist < window || key < keep);
        pr[m][r] = seen ? s[m][r] : -INFINITY;
        mx = fmaxf(mx, pr[m][r]);
      }
      mx = col4_max(mx);
      const float m_new = fmaxf(mrun[m], mx), ms = m_new == -INFINITY ? 0.f : m_new;
      al[m] = __builtin_amdgcn_exp2f(mrun[m] - ms);                       // (nothing seen yet: exp2(-inf) = 0)
      mrun[m] = m_new;
      float sum = 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        pr[m][r] = __builtin_amdgcn_exp2f(pr[m][r] - ms);
        sum += pr[m][r];
      }
      if (m_new == -INFINITY) al[m] = 1.f;
      lrun[m] = fmaf(lrun[m], al[m], sum);                                // (this lane's keys only; summed over the column at the end)
    }
    if (__any(al[0] != 1.f || al[1] != 1.f)) {
#pragma unroll
      for (int m = 0; m < 2; ++m)
#pragma unroll
        for (int b = 0; b < NB; ++b) acc[m][b] *= al[m];
    }
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int b = 0; b < NB; ++b) {
        acc[0][b] = __builtin_amdgcn_mfma_f32_16x16x4f32(v[r][b], pr[0][r], acc[0][b], 0, 0, 0);
        acc[1][b] = __builtin_amdgcn_mfma_f32_16x16x4f32(v[r][b], pr[1][r], acc[1][b], 0, 0, 0);
      }
    j += NW;
    if (j >= kept_tiles && j < first_tile) j += (first_tile - j + NW - 1) / NW * NW;
  }
  // merge: common maximum per column, every wave's sums scaled to it and added in wave order
  float ltot[2];
#pragma unroll
  for (int m = 0; m < 2; ++m) {
    lrun[m] = col4_sum(lrun[m]);
    if (g == 0) {
      ml[((wave * 2 + m) * QC + r16) * 2] = mrun[m];
      ml[((wave * 2 + m) * QC + r16) * 2 + 1] = lrun[m];
    }
  }
  __syncthreads();
#pragma unroll
  for (int m = 0; m < 2; ++m) {
    float M = -INFINITY;
    for (int w = 0; w < NW; ++w) M = fmaxf(M, ml[((w * 2 + m) * QC + r16) * 2]);
    const float ms = M == -INFINITY ? 0.f : M;
    float l = 0.f;
    for (int w = 0; w < NW; ++w) l = fmaf(ml[((w * 2 + m) * QC + r16) * 2 + 1], __builtin_amdgcn_exp2f(ml[((w * 2 + m) * QC + r16) * 2] - ms), l);
    ltot[m] = l > 0.f ? 1.f / l : 0.f;
    const float f = __builtin_amdgcn_exp2f(mrun[m] - ms) * ltot[m];
#pragma unroll
    for (int b = 0; b < NB; ++b) acc[m][b] *= f;
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
  // difference, norm over the head's columns, store: 16 lanes per column of the first 4 waves
  if (tid < 256) {
    const int c = tid >> 4, l16 = tid & 15;
    const float* o1 = os + c * OP;
    const float* o2 = o1 + QC * OP;
    float ss = 0.f;
    for (int i = l16; i < Dv; i += 16) {
      const float d = o1[i] - p.lambda * o2[i];
      ss = fmaf(d, d, ss);
    }
#pragma unroll
    for (int o = 8; o > 0; o >>= 1) ss += __shfl_xor(ss, o);
    if (c < ncol) {
      const float r = p.mult / sqrtf(ss / (float)Dv + p.eps);
      const long tok = decode ? t0 : t0 + c;
      const int h = decode ? h0 + c : h0;
      T* out = (T*)p.out + tok * p.ldo + (long)h * Dv;
      for (int i = l16; i < Dv; i += 16) st_f(out + i, (o1[i] - p.lambda * o2[i]) * r);
    }
  }
}

size_t lds_bytes(const vlm_diff_attn_args& a, int NB, int NW) {
  const int QP = ((a.D + 15) & ~15) + 4;
  return ((size_t)2 * QC * QP + (size_t)NW * 2 * QC * 2 + (size_t)2 * QC * (NB * 16 + 4)) * sizeof(float);
}

template <typename T, int NW>
int launch(const vlm_diff_attn_args& a, dim3 grid, int decode, int hpb, hipStream_t st) {
  const int need = (a.Dv + 15) / 16;
  const int NB = need <= 1 ? 1 : need <= 2 ? 2 : need <= 4 ? 4 : need <= 8 ? 8 : 16;
  const size_t lds = lds_bytes(a, NB, NW);
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
  if (bad(a) || rows < 0) return VLM_ERR_ARG;
  const int R = a->H / a->KH, hpb = R < 16 ? R : 16;
  const long gy = (long)a->KH * ((R + hpb - 1) / hpb);
  if (gy > 65535) return VLM_ERR_SHAPE;
  if (rows == 0) return VLM_OK;
  const dim3 grid(rows, (unsigned)gy);
  return dtype ? launch<float, 4>(*a, grid, 1, hpb, (hipStream_t)stream) : launch<bf16_t, 4>(*a, grid, 1, hpb, (hipStream_t)stream);
}
