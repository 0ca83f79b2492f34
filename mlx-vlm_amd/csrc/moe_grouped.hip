// Mixture of gated experts for prompts: only the (token, expert) pairs that the router chose are evaluated.  The rows of an expert stand side by
// side ("slots": expert 0's tokens in order, padded to whole tiles of 128, expert 1's, ...), so that a tile of the products belongs to one
// expert:
//
//   vlm_moe_plan          gate table fp32 [T][E] (0: not chosen) -> slot tables: tok [cap] (the slot's token, -1: padding), tile_expert [cap / 128],
//                         ntiles, and per token its slots in expert order (slots [T][top], -1: fewer); count [E]: scratch
//   vlm_moe_grouped_up    act[slot] = act(W_gate,e h[tok]) * (W_up,e h[tok]) * gate[tok][e]: gathered rows, both products and the activation in one
//                         kernel.  W: expert e's rows [gate_e | up_e], 2 ff rows side by side
//   vlm_moe_grouped_down  y[slot] = W_down,e act[slot]; W: the experts' columns side by side ([N][E ff])
//
// The sum over a token's slots belongs to the reader (vlm_sandwich_step reads them).  bf16, fp32 sums; K of both products a multiple of 64.
//
// Products: 128 x 128 tile, 64 k deep, 4 waves (2 x 2) of v_mfma_f32_16x16x32_bf16; tiles arrive by LDS-DMA (global_load_lds, 16 bytes per lane) in two
// buffers, 16-byte pieces swizzled with the row on the source side so that the operand reads of 16 lanes fall into different banks; gathered rows
// are nothing but other source addresses.  D^T = W A^T: a lane ends with 4 neighbouring columns of one row.
#include "common.hpp"
#include "../../include/vlm_hip.h"

namespace {

constexpr int BM = 128, BN = 128, BK = 64, ROWB = BK * 2, STAGE = (BM + BN) * ROWB;

__device__ __forceinline__ int lds_off(int row, int slot) { return row * ROWB + ((slot ^ ((row >> 1) & 7)) << 4); }

// grid (E): tokens of every expert; token slots marked empty
__global__ __launch_bounds__(1024) void moe_count_kernel(const float* __restrict__ gate, int T, int E, int top, int* __restrict__ count,
                                                         int* __restrict__ slots) {
  __shared__ int part[16];
  const int tid = threadIdx.x, e = blockIdx.x;
  int n = 0;
  for (int t = tid; t < T; t += 1024) n += gate[(long)t * E + e] != 0.f;
  for (int i = e * 1024 + tid; i < T * top; i += E * 1024) slots[i] = -1;
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) n += __shfl_xor(n, o);
  if ((tid & 63) == 0) part[tid >> 6] = n;
  __syncthreads();
  if (tid == 0) {
    int s = 0;
    for (int w = 0; w < 16; ++w) s += part[w];
    count[e] = s;
  }
}

// grid (E): the expert's first slot from the counts of those before it, then its tokens in order, 1024 at a time
__global__ __launch_bounds__(1024) void moe_place_kernel(const float* __restrict__ gate, int T, int E, int top, const int* __restrict__ count,
                                                         int* __restrict__ tok, int* __restrict__ tile_expert, int* __restrict__ ntiles,
                                                         int* __restrict__ slots) {
  __shared__ int part[16], before[16];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, e = blockIdx.x;
  int b = 0;
  for (int f = tid; f < e; f += 1024) b += (count[f] + BM - 1) / BM * BM;
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) b += __shfl_xor(b, o);
  if (lane == 0) before[wave] = b;
  __syncthreads();
  int at = 0;
  for (int w = 0; w < 16; ++w) at += before[w];
  const int n = count[e], end = at + (n + BM - 1) / BM * BM;
  if (e == E - 1 && tid == 0) *ntiles = end / BM;
  for (int i = at / BM + tid; i < end / BM; i += 1024) tile_expert[i] = e;
  for (int i = at + n + tid; i < end; i += 1024) tok[i] = -1;
  for (int t0 = 0; t0 < T; t0 += 1024) {
    const int t = t0 + tid;
    const bool mine = t < T && gate[(long)min(t, T - 1) * E + e] != 0.f;
    const unsigned long long m = __ballot(mine);
    if (lane == 0) part[wave] = __popcll(m);
    __syncthreads();
    int ahead = 0, total = 0;
    for (int w = 0; w < 16; ++w) {
      if (w < wave) ahead += part[w];
      total += part[w];
    }
    if (mine) {
      const int slot = at + ahead + __popcll(m & ((1ull << lane) - 1ull));
      int k = 0;                                         // how many experts before this one the token chose
      for (int f = 0; f < e; ++f) k += gate[(long)t * E + f] != 0.f;
      tok[slot] = t;
      if (k < top) slots[(long)t * top + k] = slot;
    }
    at += total;
    __syncthreads();
  }
}

__device__ __forceinline__ float expert_act(float g, float u, int act, float limit) {
  if (act == 3) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g * sigmoidf_(1.702f * g) * (u + 1.f);
  }
  if (act == 1) return g * sigmoidf_(g) * u;
  return 0.5f * g * (1.0f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g))) * u;
}

// UP: rows gathered by token, W tile = 64 gate and 64 up rows in alternating groups of 16; else rows as they stand, W tile = 128 rows
template <bool UP>
__global__ __launch_bounds__(256) void moe_grouped_kernel(vlm_moe_grouped_args p, int tiles_n, int row_tiles, int nwg) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  // workgroups with the same (id % 8) share an L2: each of the 8 walks a contiguous range, row tiles of one column tile first
  int bid = blockIdx.x;
  {
    const int q = nwg >> 3, r = nwg & 7, xcd = bid & 7, idx = bid >> 3;
    bid = (xcd < r ? xcd * (q + 1) : r * (q + 1) + (xcd - r) * q) + idx;
  }
  const int pn = bid / row_tiles, pm = bid - pn * row_tiles;
  if (pm >= *p.ntiles) return;
  const int e = p.tile_expert[pm], m0 = pm * BM, K = p.K, ff = p.ff;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), wm = wave >> 1, wn = wave & 1;
  const bf16_t* A = (const bf16_t*)p.a;
  const bf16_t* W = (const bf16_t*)p.w + (UP ? (long)e * 2 * ff * p.ldw : (long)e * ff);
  const int rl = lane >> 3, sp = lane & 7;
  const bf16_t *asrc[4], *wsrc[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int row = 8 * (wave * 4 + j) + rl, sw = (sp ^ ((row >> 1) & 7)) << 3;
    long ar = m0 + row;
    if (UP) ar = max(p.tok[m0 + row], 0);                // (a padding slot reads some row; its result is not used)
    asrc[j] = A + ar * p.lda + sw;
    int wr;
    if (UP) wr = min(pn * 64 + (row >> 5) * 16 + (row & 15), ff - 1) + ((row >> 4) & 1) * ff;
    else wr = min(pn * BN + row, p.N - 1);
    wsrc[j] = W + (long)wr * p.ldw + sw;
  }
  auto issue = [&](int kt, int buf) {
    char* as = smem + buf * STAGE;
    char* ws = as + BM * ROWB;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(asrc[j] + (long)kt * BK),
                                       (__attribute__((address_space(3))) void*)(as + (wave * 4 + j) * 1024), 16, 0, 0);
#pragma unroll
    for (int j = 0; j < 4; ++j)
      __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(wsrc[j] + (long)kt * BK),
                                       (__attribute__((address_space(3))) void*)(ws + (wave * 4 + j) * 1024), 16, 0, 0);
  };
  f32x4_t acc[4][4];                                     // [W tile][A tile]
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  const int nk = K / BK, r16 = lane & 15, g = lane >> 4;
  issue(0, 0);
  __syncthreads();                                       // (drains the DMA in flight)
  for (int kt = 0; kt < nk; ++kt) {
    if (kt + 1 < nk) issue(kt + 1, (kt + 1) & 1);
    const char* as = smem + (kt & 1) * STAGE;
    const char* ws = as + BM * ROWB;
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      bf16x8_t af[4], wf[4];
      const int slot = ks * 4 + g;
#pragma unroll
      for (int j = 0; j < 4; ++j) af[j] = *reinterpret_cast<const bf16x8_t*>(as + lds_off(wm * 64 + j * 16 + r16, slot));
#pragma unroll
      for (int i = 0; i < 4; ++i) wf[i] = *reinterpret_cast<const bf16x8_t*>(ws + lds_off(wn * 64 + i * 16 + r16, slot));
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[i], af[j], acc[i][j], 0, 0, 0);
    }
    __syncthreads();
  }
  // the result tile goes through LDS (free now) and out in whole 16-byte pieces
  constexpr int OUT_N = UP ? 64 : 128, LD = OUT_N + 8;
  bf16_t* cs = reinterpret_cast<bf16_t*>(smem);
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int ml = wm * 64 + j * 16 + r16;
    if constexpr (UP) {
      const int t = p.tok[m0 + ml];
      const float r = t < 0 ? 0.f : p.gate[(long)t * p.E + e];
#pragma unroll
      for (int i = 0; i < 4; i += 2) {                   // W tiles 2 x, 2 x + 1: gate and up of the same 16 columns
        float v[4];
#pragma unroll
        for (int k = 0; k < 4; ++k) v[k] = expert_act(acc[i][j][k], acc[i + 1][j][k], p.act, p.limit) * r;
        *reinterpret_cast<uint2*>(cs + ml * LD + wn * 32 + (i / 2) * 16 + 4 * g) = make_uint2(pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3]));
      }
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        *reinterpret_cast<uint2*>(cs + ml * LD + wn * 64 + i * 16 + 4 * g) = make_uint2(pack_bf2(acc[i][j][0], acc[i][j][1]), pack_bf2(acc[i][j][2], acc[i][j][3]));
    }
  }
  __syncthreads();
  const int n_out = UP ? ff : p.N, n0 = pn * OUT_N;
  for (int i = tid; i < BM * (OUT_N / 8); i += 256) {
    const int row = i / (OUT_N / 8), c = (i % (OUT_N / 8)) * 8;
    if (n0 + c < n_out && p.tok[m0 + row] >= 0)
      *reinterpret_cast<uint4*>((bf16_t*)p.out + (long)(m0 + row) * p.ldo + n0 + c) = *reinterpret_cast<const uint4*>(cs + row * LD + c);
  }
}

template <bool UP> int grouped(const vlm_moe_grouped_args* a, int row_tiles, void* stream) {
  if (!a || !a->a || !a->w || !a->tok || !a->tile_expert || !a->ntiles || !a->out || a->E <= 0 || a->ff <= 0 || a->K <= 0 || row_tiles < 0 ||
      a->lda < a->K || (UP ? !a->gate || a->ldw < a->K || a->ldo < a->ff || a->act < 0 || a->act > 3 || a->act == 2 || (a->act == 3 && !(a->limit >= 0.f))
                           : a->N <= 0 || a->K != a->ff || a->ldw < (long)a->E * a->ff || a->ldo < a->N))
    return VLM_ERR_ARG;
  if (a->K % 64 || a->ff % 8 || (!UP && a->N % 8) || a->lda % 8 || a->ldw % 8 || a->ldo % 8 ||
      (((uintptr_t)a->a | (uintptr_t)a->w | (uintptr_t)a->out) & 15))
    return VLM_ERR_SHAPE;
  if (row_tiles == 0) return VLM_OK;
  const int tiles_n = UP ? (a->ff + 63) / 64 : (a->N + BN - 1) / BN;
  const long nwg = (long)tiles_n * row_tiles;
  if (nwg > 0x7fffffff) return VLM_ERR_SHAPE;
  constexpr int lds = 2 * STAGE;                         // 64 KiB
  hipError_t err = hipFuncSetAttribute((const void*)moe_grouped_kernel<UP>, hipFuncAttributeMaxDynamicSharedMemorySize, lds);
  if (err != hipSuccess) return VLM_ERR_HIP + (int)err;
  hipLaunchKernelGGL((moe_grouped_kernel<UP>), dim3((unsigned)nwg), dim3(256), lds, (hipStream_t)stream, *a, tiles_n, row_tiles, (int)nwg);
  VLM_CHECK_LAUNCH();
  return VLM_OK;
}

}  // namespace

extern "C" int vlm_moe_plan(const void* gate, int T, int E, int top, int cap, void* count, void* tok, void* tile_expert, void* ntiles, void* slots,
                            void* stream) {
  if (!gate || !count || !tok || !tile_expert || !ntiles || !slots || T <= 0 || E <= 0 || top <= 0 ||
      (long)cap < ((long)T * top + BM - 1) / BM * BM + (long)E * BM)
    return VLM_ERR_ARG;
  if (E > 256 || (long)T * top > 0x3fffffff) return VLM_ERR_SHAPE;
  hipStream_t st = (hipStream_t)stream;
  hipLaunchKernelGGL(moe_count_kernel, dim3(E), dim3(1024), 0, st, (const float*)gate, T, E, top, (int*)count, (int*)slots);
  VLM_CHECK_LAUNCH();
  hipLaunchKernelGGL(moe_place_kernel, dim3(E), dim3(1024), 0, st, (const float*)gate, T, E, top, (const int*)count, (int*)tok, (int*)tile_expert,
                     (int*)ntiles, (int*)slots);
  VLM_CHECK_LAUNCH();
  return VLM_OK;
}

extern "C" int vlm_moe_grouped_up(const vlm_moe_grouped_args* a, int row_tiles, void* stream) { return grouped<true>(a, row_tiles, stream); }
extern "C" int vlm_moe_grouped_down(const vlm_moe_grouped_args* a, int row_tiles, void* stream) { return grouped<false>(a, row_tiles, stream); }
