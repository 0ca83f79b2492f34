// Latent attention (see latent_attn.hip: absorbed form, ONE cached row [c (R) | kr (Dr)] per token, scores over R + Dr, values = c) on the
// bf16 matrix cores, for bf16 queries and bf16 pools whose rows come in whole 16-byte pieces (R % 8 == 0, Dr % 8 == 0; R <= 512,
// R + Dr <= 576).
//
//     s_hj = scale * (q_h . row_j)        o_h = sum_j exp(s_hj) c_j / (exp(sink_h) + sum_j exp(s_hj)) (* sigmoid(gate_h))
//     j visible from i  <=>  0 <= i - j < window  (window <= 0: every j <= i); no sink: without the first term of the denominator
//
// Scores are fp32 sums, the softmax runs in fp32, and its weights enter the product with the values as two bf16 values each ((p_hi + p_lo) c),
// so nothing of a score or a weight is rounded to 8 bits.  Layout of the transposed products: attn_mfma.hpp.
//
//   blocks (prompt)  workgroup = up to 16 consecutive tokens of one sequence x 4 heads, one head per wave.  A wave keeps its 16 query
//                    columns in registers (operand layout) and the whole read-out of R columns; the key tile - one page of 64 rows,
//                    which all heads share - goes through LDS in two buffers, the next page's loads in flight while this one is
//                    used, one barrier per tile.  The same LDS rows serve as keys (16 bytes of one row per lane) and as values
//                    (8 columns of 8 keys per lane, interleaved in registers).  No exchange between the waves.
//   rows (decode)    workgroup = one token x up to 16 heads, one page at a time through LDS: the waves share the page's keys for the scores,
//                    exchange them, and share the value columns for the read-out; `nsplit` workgroups take turns over the pages, a second
//                    kernel merges their results.
#include "common.hpp"
#include "../../include/vlm_hip.h"
#include "recurrence_finish.hpp"
#include "attn_mfma.hpp"

namespace {

constexpr int PAGE = 64, QC = 16;
constexpr float LOG2E = 1.4426950408889634f;

// a key tile in LDS: rows of 32 NKS columns (zeros behind R + Dr) at an odd number of 16-byte pieces, so that the same piece of 16 neighbouring
// rows sits in different banks; one more piece behind the tile takes the stores of lanes without a piece
template <int NKS> struct Tile {
  static constexpr int PITCH = 8 * ((4 * NKS) | 1), SIZE = PAGE * PITCH + 8;
};

// 16 query columns as operands: lane (r16, g) holds dimensions 32 s + 8 g .. + 8 of column r16
template <int NKS> __device__ __forceinline__ void load_queries(const bf16_t* qrow, bool live, int Dk, int g, bf8* q) {
#pragma unroll
  for (int s = 0; s < NKS; ++s) {
    const int d = 32 * s + 8 * g;
    q[s] = zero8();
    if (live && d < Dk) q[s] = *reinterpret_cast<const bf8*>(qrow + d);
  }
}

// copies of a page's rows into a tile by 256 threads: this thread's pieces are tid, tid + 256, ... (a page's rows are contiguous in memory);
// rows past the last key repeat its last piece (they are masked)
template <int NKS> struct Stager {
  static constexpr int HALF = NKS / 2;                   // a page goes through the registers in two halves
  int loff[NKS], pieces, D8;
  u32x4_t st[HALF];
  __device__ __forceinline__ void init(bf16_t* tiles, int ntiles, int Dk, int tid) {
    D8 = Dk / 8;
    pieces = PAGE * D8;
#pragma unroll
    for (int i = 0; i < NKS; ++i) {
      const int idx = tid + 256 * i;
      loff[i] = idx < pieces ? (idx / D8) * Tile<NKS>::PITCH + (idx % D8) * 8 : PAGE * Tile<NKS>::PITCH;
    }
    const int pad = 4 * NKS - D8;                        // pieces of zeros behind every row
    for (int i = tid; i < ntiles * PAGE * pad; i += 256) {
      const int row = (i / pad) % PAGE;
      *reinterpret_cast<u32x4_t*>(tiles + (i / (pad * PAGE)) * Tile<NKS>::SIZE + row * Tile<NKS>::PITCH + (D8 + i % pad) * 8) = u32x4_t{0u, 0u, 0u, 0u};
    }
  }
  template <int H> __device__ __forceinline__ void load(const bf16_t* page, int keys, int tid) {
    const u32x4_t* src = reinterpret_cast<const u32x4_t*>(page);
    const int have = min(pieces, keys * D8) - 1;
#pragma unroll
    for (int i = 0; i < HALF; ++i) st[i] = src[min(tid + 256 * (H * HALF + i), have)];
  }
  template <int H> __device__ __forceinline__ void store(bf16_t* tile) {
#pragma unroll
    for (int i = 0; i < HALF; ++i) *reinterpret_cast<u32x4_t*>(tile + loff[H * HALF + i]) = st[i];
  }
};

// softmax update of one query column over N scores per lane (scores in log2 units); returns the factor of what was summed before
template <int N>
__device__ __forceinline__ float softmax_update(float* pr, float& mrun, float& lrun) {
  float mx = pr[0];
#pragma unroll
  for (int i = 1; i < N; ++i) mx = fmaxf(mx, pr[i]);
  mx = col4_max(mx);
  const float m_new = fmaxf(mrun, mx), ms = m_new == -INFINITY ? 0.f : m_new;
  const float al = m_new == -INFINITY ? 1.f : __builtin_amdgcn_exp2f(mrun - ms);
  mrun = m_new;
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < N; ++i) {
    pr[i] = __builtin_amdgcn_exp2f(pr[i] - ms);
    sum += pr[i];
  }
  lrun = fmaf(lrun, al, sum);
  return al;
}

// O^T += V^T P^T for 32 keys and 128 value columns: rows of this lane's 8 keys, 8 columns each (16 bytes)
__device__ __forceinline__ void accumulate128(const u32x4_t* v, bf8 ph, bf8 pl, f32x4_t* acc) {
  bf8 vt[8];
#pragma unroll
  for (int b = 0; b < 8; ++b) {
    u32x4_t t;
#pragma unroll
    for (int i = 0; i < 4; ++i) t[i] = pair_cols(v[2 * i][b / 2], v[2 * i + 1][b / 2], b & 1);
    vt[b] = __builtin_bit_cast(bf8, t);
    acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt[b], pl, acc[b], 0, 0, 0);
  }
#pragma unroll
  for (int b = 0; b < 8; ++b) acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt[b], ph, acc[b], 0, 0, 0);
  // the interleaving of the next column runs beside a product
#pragma unroll
  for (int b = 0; b < 8; ++b) {
    __builtin_amdgcn_sched_group_barrier(0x2, 4, 0);     // VALU
    __builtin_amdgcn_sched_group_barrier(0x8, 1, 0);     // MFMA
  }
  __builtin_amdgcn_sched_group_barrier(0x8, 8, 0);
}
// this lane's pieces of 8 keys (the contraction order of 32 keys from row `key0` on) at the columns from `cols` on
__device__ __forceinline__ void load_values(const bf16_t* tile, int pitch, int key0, int cols, int r16, int g, u32x4_t* v) {
#pragma unroll
  for (int i = 0; i < 8; ++i) v[i] = *reinterpret_cast<const u32x4_t*>(tile + (key0 + 16 * (i / 4) + 4 * g + i % 4) * pitch + cols + r16 * 8);
}

__device__ __forceinline__ float head_gate(const vlm_latent_mfma_args& p, long tok, int h) {
  return p.gate ? 1.f / (1.f + expf(-bf2f(((const bf16_t*)p.gate)[tok * p.ldgate + h]))) : 1.f;
}

// NKS: 32-dimension steps of the scores, NVC: 128-column chunks of the values
template <int NKS, int NVC>
__global__ __launch_bounds__(256, 1) void latent_block_mfma_kernel(vlm_latent_mfma_args p) {
  constexpr int KP = Tile<NKS>::PITCH, TS = Tile<NKS>::SIZE;
  extern __shared__ __align__(16) bf16_t tile[];         // [2][TS]
  const int R = p.R, Dk = p.R + p.Dr;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, r16 = lane & 15, g = lane >> 4;
  const int blk = gridDim.y - 1 - blockIdx.y;            // (the blocks of a prompt's end have the most keys: they start first)
  const int t0 = p.qb_start[blk], nq = p.qb_count[blk], h = blockIdx.x * 4 + wave;
  const bool live = h < p.H;                             // (a wave without a head still helps with the loads)
  const int* bt = p.block_table + (long)p.tok_seq[t0] * p.max_pages;
  const int pos0 = p.tok_pos[t0], last = pos0 + nq - 1, mypos = r16 < nq ? pos0 + r16 : -1, window = p.window;
  const float sc = p.scale * LOG2E;
  const bf16_t* pool = (const bf16_t*)p.pool;
  const int first = window > 0 ? max(0, pos0 - window + 1) / PAGE : 0, tiles = last / PAGE + 1;
  Stager<NKS> sg;
  sg.init(tile, 2, Dk, tid);
  sg.template load<0>(pool + (long)bt[first] * PAGE * Dk, last - first * PAGE + 1, tid);
  bf8 q[NKS];
  load_queries<NKS>((const bf16_t*)p.q + ((long)(t0 + r16) * p.H + h) * Dk, live && r16 < nq, Dk, g, q);
  f32x4_t acc[NVC][8];
#pragma unroll
  for (int c = 0; c < NVC; ++c)
#pragma unroll
    for (int b = 0; b < 8; ++b) acc[c][b] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float mrun = -INFINITY, lrun = 0.f;
  sg.template store<0>(tile);
  sg.template load<1>(pool + (long)bt[first] * PAGE * Dk, last - first * PAGE + 1, tid);
  sg.template store<1>(tile);
  for (int j = first; j < tiles; ++j) {
    const bf16_t* cur = tile + ((j - first) & 1) * TS;
    bf16_t* nxt = tile + ((j + 1 - first) & 1) * TS;
    const bool more = j + 1 < tiles;
    const bf16_t* npage = pool + (long)bt[more ? j + 1 : j] * PAGE * Dk;
    const int nkeys = last - (j + 1) * PAGE + 1;
    __syncthreads();                                     // the tile is written, and everybody is through with the other buffer
    if (more) sg.template load<0>(npage, nkeys, tid);
    // scores: two k steps of the four 16-key groups per batch, the next batch's reads ahead of this one's products
    f32x4_t s[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) s[u] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    bf8 ka[2][8];
    auto keys = [&](int b, bf8* k) {
#pragma unroll
      for (int i = 0; i < 8; ++i) k[i] = *reinterpret_cast<const bf8*>(cur + (16 * (i & 3) + r16) * KP + 32 * (2 * b + i / 4) + 8 * g);
    };
    keys(0, ka[0]);
#pragma unroll
    for (int b = 0; b < NKS / 2; ++b) {
      if (b + 1 < NKS / 2) keys(b + 1, ka[(b + 1) & 1]);
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int i = 0; i < 8; ++i) s[i & 3] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ka[b & 1][i], q[2 * b + i / 4], s[i & 3], 0, 0, 0);
      __builtin_amdgcn_sched_barrier(0);
    }
    u32x4_t v[2][8];
    load_values(cur, KP, 0, 0, r16, g, v[0]);            // (in flight during the softmax)
    __builtin_amdgcn_sched_barrier(0);
    const int lo = j * PAGE;
    float pr[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) pr[i] = s[i / 4][i % 4] * sc;
    if (!(lo + PAGE - 1 <= pos0 && (window <= 0 || last - lo < window))) {
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int dist = mypos - (lo + 16 * (i / 4) + 4 * g + i % 4);
        if (!(dist >= 0 && (window <= 0 || dist < window))) pr[i] = -INFINITY;
      }
    }
    const float al = softmax_update<16>(pr, mrun, lrun);
    if (__any(al != 1.f)) {
#pragma unroll
      for (int c = 0; c < NVC; ++c)
#pragma unroll
        for (int b = 0; b < 8; ++b) acc[c][b] *= al;
    }
    if (more) {
      sg.template store<0>(nxt);
      sg.template load<1>(npage, nkeys, tid);
    }
    bf8 ph[2], pl[2];
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) split8(pr + 8 * kk, ph[kk], pl[kk]);
#pragma unroll
    for (int i = 0; i < 2 * NVC; ++i) {                  // 32 keys x 128 columns at a time, the next piece's reads ahead
      if (i + 1 < 2 * NVC) load_values(cur, KP, 32 * ((i + 1) / NVC), 128 * ((i + 1) % NVC), r16, g, v[(i + 1) & 1]);
      __builtin_amdgcn_sched_barrier(0);
      accumulate128(v[i & 1], ph[i / NVC], pl[i / NVC], acc[i % NVC]);
      __builtin_amdgcn_sched_barrier(0);
    }
    if (more) sg.template store<1>(nxt);
  }
  float l = col4_sum(lrun);
  const float ms = mrun == -INFINITY ? 0.f : mrun;
  if (!live || r16 >= nq) return;
  if (p.sink) l += __builtin_amdgcn_exp2f(p.sink[h] * LOG2E - ms);
  const float f = (l > 0.f ? 1.f / l : 0.f) * head_gate(p, t0 + r16, h);
  bf16_t* out = (bf16_t*)p.out + ((long)(t0 + r16) * p.H + h) * R;
#pragma unroll
  for (int c = 0; c < NVC; ++c)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int col = 128 * c + (4 * g + r) * 8;
      if (col < R)
        *reinterpret_cast<uint4*>(out + col) = make_uint4(pack_bf2(acc[c][0][r] * f, acc[c][1][r] * f), pack_bf2(acc[c][2][r] * f, acc[c][3][r] * f),
                                                          pack_bf2(acc[c][4][r] * f, acc[c][5][r] * f), pack_bf2(acc[c][6][r] * f, acc[c][7][r] * f));
    }
}

template <int NKS, int NVC>
__global__ __launch_bounds__(256) void latent_rows_mfma_kernel(vlm_latent_mfma_args p) {
  constexpr int KP = Tile<NKS>::PITCH, TS = Tile<NKS>::SIZE, SP = QC + 1;
  extern __shared__ __align__(16) bf16_t tile[];         // [TS], then scores fp32 [64 keys][SP]
  float* sl = reinterpret_cast<float*>(tile + TS);
  const int R = p.R, Dk = p.R + p.Dr;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, r16 = lane & 15, g = lane >> 4;
  const int t = blockIdx.x, h0 = blockIdx.y * QC, ncol = min(QC, p.H - h0), z = blockIdx.z;
  const int* bt = p.block_table + (long)p.tok_seq[t] * p.max_pages;
  const int pos = p.tok_pos[t], window = p.window;
  const int first = window > 0 ? max(0, pos - window + 1) / PAGE : 0, tiles = pos / PAGE + 1;
  const bool split = gridDim.z > 1;
  const float sc = p.scale * LOG2E;
  float* part = p.part + (((long)z * p.H + h0 + r16) * gridDim.x + t) * (R + 2);        // of this lane's column
  if (first + z >= tiles) {                              // no keys for this workgroup: only the marks of an empty part (uniform)
    if (tid < ncol) {
      part[R] = -INFINITY;
      part[R + 1] = 0.f;
    }
    return;
  }
  const bf16_t* pool = (const bf16_t*)p.pool;
  Stager<NKS> sg, sg2;                                   // (both halves of a page in flight at once)
  sg.init(tile, 1, Dk, tid);
  sg2.pieces = sg.pieces;
  sg2.D8 = sg.D8;
  bf8 q[NKS];
  load_queries<NKS>((const bf16_t*)p.q + ((long)t * p.H + h0 + r16) * Dk, r16 < ncol, Dk, g, q);
  f32x4_t acc[8];
#pragma unroll
  for (int b = 0; b < 8; ++b) acc[b] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float mrun = -INFINITY, lrun = 0.f;
  for (int j = first + z; j < tiles; j += gridDim.z) {
    const bf16_t* page = pool + (long)bt[j] * PAGE * Dk;
    sg.template load<0>(page, pos - j * PAGE + 1, tid);
    sg2.template load<1>(page, pos - j * PAGE + 1, tid);
    __syncthreads();                                     // (everybody is through with the previous page and its scores)
    sg.template store<0>(tile);
#pragma unroll
    for (int i = 0; i < NKS / 2; ++i) *reinterpret_cast<u32x4_t*>(tile + sg.loff[NKS / 2 + i]) = sg2.st[i];
    __syncthreads();
    f32x4_t s = {0.f, 0.f, 0.f, 0.f};                    // keys 16 wave + 4 g + r of the page
#pragma unroll
    for (int k = 0; k < NKS; ++k)
      s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf8*>(tile + (16 * wave + r16) * KP + 32 * k + 8 * g), q[k], s, 0, 0, 0);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int key = 16 * wave + 4 * g + r, dist = pos - (j * PAGE + key);
      sl[key * SP + r16] = dist >= 0 && (window <= 0 || dist < window) ? s[r] * sc : -INFINITY;
    }
    __syncthreads();
    float pr[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) pr[i] = sl[(16 * (i / 4) + 4 * g + i % 4) * SP + r16];
    const float al = softmax_update<16>(pr, mrun, lrun); // (the same in every wave)
    if (wave < NVC) {
#pragma unroll
      for (int b = 0; b < 8; ++b) acc[b] *= al;
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        bf8 ph, pl;
        split8(pr + 8 * kk, ph, pl);
        u32x4_t v[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] = *reinterpret_cast<const u32x4_t*>(tile + (32 * kk + 16 * (i / 4) + 4 * g + i % 4) * KP + 128 * wave + r16 * 8);
        accumulate128(v, ph, pl, acc);
      }
    }
  }
  float l = col4_sum(lrun);
  if (r16 >= ncol) return;
  const int h = h0 + r16;
  const float ms = mrun == -INFINITY ? 0.f : mrun;
  if (split) {
    if (wave == 0 && g == 0) {
      part[R] = mrun;
      part[R + 1] = l;
    }
  } else if (p.sink) {
    l += __builtin_amdgcn_exp2f(p.sink[h] * LOG2E - ms);
  }
  if (wave >= NVC) return;
  const float f = split ? 1.f : (l > 0.f ? 1.f / l : 0.f) * head_gate(p, t, h);
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int col = 128 * wave + (4 * g + r) * 8;
    if (col >= R) continue;
    if (split) {                                         // (R is even and a part's rows are R + 2 long: 8-byte aligned)
#pragma unroll
      for (int b = 0; b < 8; b += 2) *reinterpret_cast<float2*>(part + col + b) = make_float2(acc[b][r], acc[b + 1][r]);
    } else {
      *reinterpret_cast<uint4*>((bf16_t*)p.out + ((long)t * p.H + h) * R + col) =
          make_uint4(pack_bf2(acc[0][r] * f, acc[1][r] * f), pack_bf2(acc[2][r] * f, acc[3][r] * f), pack_bf2(acc[4][r] * f, acc[5][r] * f),
                     pack_bf2(acc[6][r] * f, acc[7][r] * f));
    }
  }
}

// merge of the splits' partial results: grid (rows, H, chunks of 256 columns).  part: [split][H][rows][R sums | maximum | sum]; the splits
// that had keys come first
__global__ __launch_bounds__(256) void latent_merge_kernel(vlm_latent_mfma_args p, int nsplit) {
  const long t = blockIdx.x;
  const int h = blockIdx.y, lane = threadIdx.x & 63, R = p.R;
  const long step = (long)p.H * gridDim.x * (R + 2);
  const float* q = p.part + ((long)h * gridDim.x + t) * (R + 2);
  const float M_mine = lane < nsplit ? q[lane * step + R] : -INFINITY, l_mine = lane < nsplit ? q[lane * step + R + 1] : 0.f;
  const float M = wave_max(M_mine), ms = M == -INFINITY ? 0.f : M;
  const float f_mine = __builtin_amdgcn_exp2f(M_mine - ms);
  float l = wave_sum(l_mine * f_mine);
  if (p.sink) l += __builtin_amdgcn_exp2f(p.sink[h] * LOG2E - ms);
  const float inv = (l > 0.f ? 1.f / l : 0.f) * head_gate(p, t, h);
  const int n = __popcll(__ballot(M_mine != -INFINITY));
  const int c = min(blockIdx.z * 256 + (int)threadIdx.x, R - 1);          // (whole waves: the shuffles below need every lane)
  float a = 0.f;
  for (int z0 = 0; z0 < n; z0 += 8) {                    // eight loads in flight; splits past the last one count for nothing
    float v[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = q[min(z0 + i, n - 1) * step + c];
#pragma unroll
    for (int i = 0; i < 8; ++i) a = fmaf(__shfl(f_mine, min(z0 + i, 63)) * (z0 + i < n ? 1.f : 0.f), v[i], a);
  }
  if (blockIdx.z * 256 + (int)threadIdx.x < R) ((bf16_t*)p.out)[(t * p.H + h) * R + c] = f2bf(a * inv);
}

bool bad(const vlm_latent_mfma_args* a) {
  return !a || !a->q || !a->pool || !a->tok_seq || !a->tok_pos || !a->block_table || !a->out || a->max_pages <= 0 || a->H <= 0 || a->R <= 0 || a->Dr < 0 ||
         (a->gate && a->ldgate < a->H);
}
bool shape_ok(const vlm_latent_mfma_args* a) {
  return a->R % 8 == 0 && a->Dr % 8 == 0 && a->R <= 512 && a->R + a->Dr <= 576 && a->H <= 65535 &&
         (((uintptr_t)a->q | (uintptr_t)a->pool | (uintptr_t)a->out) & 15) == 0;
}

}  // namespace

#define LATENT_SIZES(GO)                                                        \
  do {                                                                          \
    const int Dk = a->R + a->Dr;                                                \
    if (a->R <= 128 && Dk <= 192) GO(6, 1);                                     \
    else if (a->R <= 256 && Dk <= 320) GO(10, 2);                               \
    else GO(18, 4);                                                             \
  } while (0)
#define LDS_LIMIT(K, BYTES)                                                     \
  do {                                                                          \
    if ((BYTES) > 48 * 1024) {                                                  \
      hipError_t e = hipFuncSetAttribute((const void*)(K), hipFuncAttributeMaxDynamicSharedMemorySize, (int)(BYTES)); \
      if (e != hipSuccess) return VLM_ERR_HIP + (int)e;                         \
    }                                                                           \
  } while (0)

extern "C" int vlm_latent_attn_mfma_blocks(const vlm_latent_mfma_args* a, int nblocks, void* stream) {
  if (bad(a) || !a->qb_start || !a->qb_count || nblocks < 0) return VLM_ERR_ARG;
  if (!shape_ok(a)) return VLM_ERR_SHAPE;
  if (nblocks == 0) return VLM_OK;
  if (nblocks > 65535) return VLM_ERR_SHAPE;
  const dim3 grid((a->H + 3) / 4, nblocks);
#define GO(NKS, NVC)                                                                                                        \
  do {                                                                                                                      \
    constexpr size_t lds = (size_t)2 * Tile<NKS>::SIZE * sizeof(bf16_t);                                                    \
    LDS_LIMIT((latent_block_mfma_kernel<NKS, NVC>), lds);                                                                   \
    hipLaunchKernelGGL((latent_block_mfma_kernel<NKS, NVC>), grid, dim3(256), lds, (hipStream_t)stream, *a);                \
  } while (0)
  LATENT_SIZES(GO);
#undef GO
  VLM_CHECK_LAUNCH();
  return VLM_OK;
}

extern "C" int vlm_latent_attn_mfma_rows(const vlm_latent_mfma_args* a, int rows, void* stream) {
  if (bad(a) || rows < 0 || a->nsplit < 0 || a->nsplit > 64 || (a->nsplit > 1 && !a->part)) return VLM_ERR_ARG;
  if (!shape_ok(a)) return VLM_ERR_SHAPE;
  if (rows == 0) return VLM_OK;
  const int nsplit = a->nsplit > 1 ? a->nsplit : 1;
  const dim3 grid(rows, (a->H + QC - 1) / QC, nsplit);
#define GO(NKS, NVC)                                                                                                        \
  do {                                                                                                                      \
    constexpr size_t lds = (size_t)Tile<NKS>::SIZE * sizeof(bf16_t) + PAGE * (QC + 1) * sizeof(float);                      \
    LDS_LIMIT((latent_rows_mfma_kernel<NKS, NVC>), lds);                                                                    \
    hipLaunchKernelGGL((latent_rows_mfma_kernel<NKS, NVC>), grid, dim3(256), lds, (hipStream_t)stream, *a);                 \
  } while (0)
  LATENT_SIZES(GO);
#undef GO
  VLM_CHECK_LAUNCH();
  if (nsplit > 1) {
    hipLaunchKernelGGL(latent_merge_kernel, dim3(rows, a->H, (a->R + 255) / 256), dim3(256), 0, (hipStream_t)stream, *a, nsplit);
    VLM_CHECK_LAUNCH();
  }
  return VLM_OK;
}
