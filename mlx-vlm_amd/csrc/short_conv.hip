// Short causal convolutions over time, one filter per channel, on the rows of a ragged step:
//
//     out[t][c] = (residual ? in[t][c] : 0) + bias[c] + sum_(j < taps) w[c][j] * in(t - taps + 1 + j)[c]        (then silu, act = 1)
//
// in(.) before the sequence's first token is zero.  A step brings any run of consecutive tokens of a sequence (a prompt, a
// portion, one decoded token): the taps - 1 inputs before the run live in the sequence's CARRY, fp32 [slots][taps - 1][C],
// oldest first, indexed by the same slot as the sequence's recurrent state.  A run that starts at position 0 never reads the
// carry (positions below 0 are zero by the position test), so a slot that is used again needs no clearing.
//
//   vlm_short_conv_rows    one thread per (token, channel); taps are summed oldest first with fp32 FMAs whatever the cut, so
//                          the bits of a token do not depend on how its prompt was cut
//   vlm_short_conv_carry   one thread per (segment, channel), launched after every token has read the old carry: the carry
//                          becomes the last taps - 1 inputs at the segment's end (kept entries of the old carry shift down)
//   vlm_conv_qkv_rows      the same convolution over a packed projection row [q | k | v] (parts at column offsets), fused with what an
//                          attention layer does next: rotary positions on the first rot_dims dimensions of every head of q and k
//                          (pairs (i, i + rot_dims / 2), cos and sin times `amp`), q to dense fp32 rows, k (fp32, or every coordinate as
//                          two bf16 values hi + lo) and v (T) to the paged pools of the token's sequence.  Angles are evaluated once
//                          per token and workgroup.
// Input and output rows may each be fp32 or T: a convolution over normed fp32 rows that feeds a bf16 projection, or one over a
// projection's rows that feeds a recurrence.
#include "common.hpp"
#include "../../include/vlm_hip.h"
#include "recurrence_finish.hpp"

namespace {

constexpr int MAX_TAPS = 16;

template <typename T, typename TI, typename TO>
__global__ __launch_bounds__(256) void short_conv_rows_kernel(vlm_short_conv_args p, int ntok) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  const long t = blockIdx.y;
  if (c >= p.C) return;
  const int slot = p.tok_seq[t], pos = p.tok_pos[t], taps = p.taps;
  // how many of the taps - 1 tokens before t are rows of this step (segments are runs of consecutive tokens of one sequence)
  int nin = 0;
  while (nin < taps - 1 && t - nin - 1 >= 0 && p.tok_seq[t - nin - 1] == slot) ++nin;
  const TI* in = (const TI*)p.in;
  const T* w = (const T*)p.w + (long)c * taps;
  const float* carry = p.carry + (long)slot * (taps - 1) * p.C;
  const float cur = ld_f(in + t * p.ldin + c);
  float acc = p.bias ? ld_f((const T*)p.bias + c) : 0.f;
  for (int j = 0; j < taps; ++j) {
    const int back = taps - 1 - j;                       // oldest first
    float v = 0.f;
    if (back == 0) v = cur;
    else if (pos - back >= 0) v = back <= nin ? ld_f(in + (t - back) * p.ldin + c) : carry[(long)(taps - 1 - (back - nin)) * p.C + c];
    acc = fmaf(ld_f(w + j), v, acc);
  }
  if (p.residual) acc += cur;
  if (p.act == 1) acc = acc / (1.f + expf(-acc));
  st_f((TO*)p.out + t * p.ldo + c, acc);
}

template <typename TI>
__global__ __launch_bounds__(256) void short_conv_carry_kernel(vlm_short_conv_args p, int nseg) {
  const int c = blockIdx.x * 256 + threadIdx.x, seg = blockIdx.y;
  if (c >= p.C) return;
  const int t0 = p.seg_start[seg], len = p.seg_start[seg + 1] - t0, pos0 = p.seg_pos0[seg], keep = p.taps - 1;
  float* carry = p.carry + (long)p.seg_slot[seg] * keep * p.C;
  const TI* in = (const TI*)p.in;
  float v[MAX_TAPS - 1];
#pragma unroll
  for (int i = 0; i < MAX_TAPS - 1; ++i) {
    if (i < keep) {
      const int r = len - keep + i;                      // the row of the segment that lands in entry i (negative: before the segment)
      const int pos = pos0 + r;
      v[i] = pos < 0 ? 0.f : (r >= 0 ? ld_f(in + (long)(t0 + r) * p.ldin + c) : carry[(long)(keep + r) * p.C + c]);
    }
  }
#pragma unroll
  for (int i = 0; i < MAX_TAPS - 1; ++i)
    if (i < keep) carry[(long)i * p.C + c] = v[i];
}

// grid (items / 256, token groups of TB).  Items of a token, in order: q heads, then k heads, each head as rot_dims / 2 pairs followed
// by its passing dimensions; then the value columns.  A lane keeps its item's filter and the last inputs in registers and walks the
// tokens of the group; where the sequence changes (or the group starts) it fetches the inputs before the token afresh.
// TAPS >= the filter's taps (shorter ones: leading zeros)
template <typename T, int TAPS, int TB>
__global__ __launch_bounds__(256) void conv_qkv_kernel(vlm_conv_qkv_args p, int ntok) {
  extern __shared__ __align__(16) float cs[];             // [TB][half] cos, [TB][half] sin of the tokens' positions
  __shared__ long row_s[TB];
  __shared__ int pos_s[TB], slot_s[TB], nin_s[TB];
  const int tid = threadIdx.x, half = p.rot_dims / 2, per = p.D - half, taps = p.taps;
  const long t0 = (long)blockIdx.y * TB;
  const int nt = (int)min((long)TB, ntok - t0);
  for (int i = tid; i < nt * half; i += 256) {
    const int t = i / half;
    float sn, c;
    sincosf((float)p.tok_pos[t0 + t] * p.inv_freq[i % half], &sn, &c);
    cs[i] = c * p.amp;
    cs[TB * half + i] = sn * p.amp;
  }
  if (tid < nt) {
    const long t = t0 + tid;
    const int pos = p.tok_pos[t], slot = p.tok_seq[t];
    int nin = 0;                                          // how many of the taps - 1 tokens before t are rows of this step
    while (nin < taps - 1 && t - nin - 1 >= 0 && p.tok_seq[t - nin - 1] == slot) ++nin;
    pos_s[tid] = pos;
    slot_s[tid] = slot;
    nin_s[tid] = nin;
    row_s[tid] = (long)p.block_table[(long)slot * p.max_pages + pos / 64] * 64 + pos % 64;
  }
  __syncthreads();
  const int nq = p.HQ * per, nk = p.HK * per, it = blockIdx.x * 256 + tid;
  if (it >= nq + nk + p.NV) return;
  const bool is_v = it >= nq + nk, is_q = it < nq;
  int h = 0, i = 0, col;                                  // head, place in the head's items, column of the (first) input
  if (is_v) {
    col = p.voff + it - nq - nk;
  } else {
    const int r = is_q ? it : it - nq;
    h = r / per;
    i = r % per;
    col = (is_q ? p.qoff : p.koff) + h * p.D + (i >= half ? i + half : i);
  }
  const bool pair = !is_v && i < half;
  const int D8 = (p.D + 7) & ~7;
  const T* x = (const T*)p.x + col;
  float wu[TAPS], wv[TAPS], hu[TAPS], hv[TAPS];           // filters; inputs, oldest first (the last entry: the token itself)
#pragma unroll
  for (int j = 0; j < TAPS; ++j) {
    const int f = j - (TAPS - taps);
    wu[j] = taps == 0 ? (j == TAPS - 1 ? 1.f : 0.f) : (f >= 0 ? ld_f((const T*)p.w + (long)col * taps + f) : 0.f);
    wv[j] = taps == 0 ? (j == TAPS - 1 ? 1.f : 0.f) : (f >= 0 && pair ? ld_f((const T*)p.w + (long)(col + half) * taps + f) : 0.f);
    hu[j] = hv[j] = 0.f;
  }
  for (int t = 0; t < nt; ++t) {
    const long tok = t0 + t;
    const int pos = pos_s[t], nin = nin_s[t], slot = slot_s[t];
    if (t > 0 && nin > 0) {                               // (nin > 0: the row before is the token before, or taps <= 1)
#pragma unroll
      for (int j = 0; j + 1 < TAPS; ++j) {
        hu[j] = hu[j + 1];
        hv[j] = hv[j + 1];
      }
    } else {
      const float* carry = p.carry + (long)slot * (taps > 1 ? taps - 1 : 0) * p.C + col;
#pragma unroll
      for (int j = 0; j + 1 < TAPS; ++j) {
        const int back = TAPS - 1 - j;
        const bool ok = back < taps && pos - back >= 0;
        const bool here = back <= nin;
        hu[j] = !ok ? 0.f : here ? ld_f(x + (tok - back) * p.ldx) : carry[(long)(taps - 1 - (back - nin)) * p.C];
        hv[j] = !ok || !pair ? 0.f : here ? ld_f(x + (tok - back) * p.ldx + half) : carry[(long)(taps - 1 - (back - nin)) * p.C + half];
      }
    }
    hu[TAPS - 1] = ld_f(x + tok * p.ldx);
    hv[TAPS - 1] = pair ? ld_f(x + tok * p.ldx + half) : 0.f;
    float u = 0.f, v = 0.f;
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
      u = fmaf(wu[j], hu[j], u);
      v = fmaf(wv[j], hv[j], v);
    }
    if (is_v) {
      st_f((T*)p.vpool + row_s[t] * p.NV + (it - nq - nk), u);
      continue;
    }
    if (pair) {
      const float c = cs[t * half + i], s = cs[TB * half + t * half + i], a = u;
      u = a * c - v * s;
      v = v * c + a * s;
    }
    const int d = i >= half ? i + half : i;
    if (is_q) {
      float* dst = p.q + (tok * p.HQ + h) * p.D + d;
      *dst = u;
      if (pair) dst[half] = v;
    } else if (p.k_split) {
      bf16_t* dst = (bf16_t*)p.kpool + (row_s[t] * p.HK + h) * 2 * D8 + d;
      const bf16_t uh = f2bf(u);
      dst[0] = uh;
      dst[D8] = f2bf(u - bf2f(uh));
      if (pair) {
        const bf16_t vh = f2bf(v);
        dst[half] = vh;
        dst[D8 + half] = f2bf(v - bf2f(vh));
      }
    } else {
      float* dst = (float*)p.kpool + (row_s[t] * p.HK + h) * p.D + d;
      *dst = u;
      if (pair) dst[half] = v;
    }
  }
}

template <typename T, int TAPS>
int conv_qkv_launch(const vlm_conv_qkv_args& a, int ntok, hipStream_t st) {
  const int total = (a.HQ + a.HK) * (a.D - a.rot_dims / 2) + a.NV;
  const int TB = ntok >= 1024 ? 16 : ntok >= 128 ? 4 : 1;
  const dim3 grid((total + 255) / 256, (ntok + TB - 1) / TB);
  const size_t lds = (size_t)TB * (a.rot_dims > 0 ? a.rot_dims : 1) * sizeof(float);
  if (grid.y > 65535 || lds > 48 * 1024) return VLM_ERR_SHAPE;
  if (TB == 16) hipLaunchKernelGGL((conv_qkv_kernel<T, TAPS, 16>), grid, dim3(256), lds, st, a, ntok);
  else if (TB == 4) hipLaunchKernelGGL((conv_qkv_kernel<T, TAPS, 4>), grid, dim3(256), lds, st, a, ntok);
  else hipLaunchKernelGGL((conv_qkv_kernel<T, TAPS, 1>), grid, dim3(256), lds, st, a, ntok);
  VLM_CHECK_LAUNCH();
  return VLM_OK;
}

template <typename T>
int conv_qkv_run(const vlm_conv_qkv_args& a, int ntok, hipStream_t st) {
  if (a.taps <= 1) return conv_qkv_launch<T, 1>(a, ntok, st);
  if (a.taps <= 2) return conv_qkv_launch<T, 2>(a, ntok, st);
  if (a.taps <= 3) return conv_qkv_launch<T, 3>(a, ntok, st);
  if (a.taps <= 4) return conv_qkv_launch<T, 4>(a, ntok, st);
  return conv_qkv_launch<T, MAX_TAPS>(a, ntok, st);
}

bool bad(const vlm_short_conv_args* a) {
  return !a || !a->in || !a->w || a->C <= 0 || a->taps < 1 || a->ldin < a->C || (a->taps > 1 && !a->carry) || a->act < 0 || a->act > 1;
}

}  // namespace

extern "C" int vlm_short_conv_rows(const vlm_short_conv_args* a, int ntok, int dtype, void* stream) {
  if (bad(a) || !a->out || a->ldo < a->C || !a->tok_seq || !a->tok_pos || ntok < 0) return VLM_ERR_ARG;
  if (a->taps > MAX_TAPS || ntok > 65535 * 16) return VLM_ERR_SHAPE;
  if (ntok == 0) return VLM_OK;
  dim3 grid((a->C + 255) / 256, ntok);
  hipStream_t st = (hipStream_t)stream;
#define GO(T, TI, TO) hipLaunchKernelGGL((short_conv_rows_kernel<T, TI, TO>), grid, dim3(256), 0, st, *a, ntok)
  if (dtype) GO(float, float, float);
  else if (a->in_f32 && a->out_f32) GO(bf16_t, float, float);
  else if (a->in_f32) GO(bf16_t, float, bf16_t);
  else if (a->out_f32) GO(bf16_t, bf16_t, float);
  else GO(bf16_t, bf16_t, bf16_t);
#undef GO
  VLM_CHECK_LAUNCH();
  return VLM_OK;
}

extern "C" int vlm_short_conv_carry(const vlm_short_conv_args* a, int nseg, int dtype, void* stream) {
  if (bad(a) || !a->seg_start || !a->seg_slot || !a->seg_pos0 || nseg < 0) return VLM_ERR_ARG;
  if (a->taps > MAX_TAPS || nseg > 65535) return VLM_ERR_SHAPE;
  if (nseg == 0 || a->taps == 1) return VLM_OK;
  dim3 grid((a->C + 255) / 256, nseg);
  hipStream_t st = (hipStream_t)stream;
  if (dtype || a->in_f32) hipLaunchKernelGGL(short_conv_carry_kernel<float>, grid, dim3(256), 0, st, *a, nseg);
  else hipLaunchKernelGGL(short_conv_carry_kernel<bf16_t>, grid, dim3(256), 0, st, *a, nseg);
  VLM_CHECK_LAUNCH();
  return VLM_OK;
}

extern "C" int vlm_conv_qkv_rows(const vlm_conv_qkv_args* a, int ntok, int dtype, void* stream) {
  if (!a || !a->x || !a->q || !a->kpool || !a->vpool || !a->tok_seq || !a->tok_pos || !a->block_table || a->max_pages <= 0 || ntok < 0 ||
      a->HQ <= 0 || a->HK <= 0 || a->D <= 0 || a->NV <= 0 || a->taps < 0 || (a->taps > 0 && !a->w) || (a->taps > 1 && !a->carry) ||
      a->rot_dims < 0 || (a->rot_dims & 1) || a->rot_dims > a->D || (a->rot_dims && !a->inv_freq) || a->ldx < a->C || a->qoff < 0 ||
      a->koff < 0 || a->voff < 0 || a->qoff + (long)a->HQ * a->D > a->C || a->koff + (long)a->HK * a->D > a->C || a->voff + (long)a->NV > a->C)
    return VLM_ERR_ARG;
  if (a->k_split && dtype) return VLM_ERR_ARG;
  if (a->taps > MAX_TAPS) return VLM_ERR_SHAPE;
  if (ntok == 0) return VLM_OK;
  return dtype ? conv_qkv_run<float>(*a, ntok, (hipStream_t)stream) : conv_qkv_run<bf16_t>(*a, ntok, (hipStream_t)stream);
}
