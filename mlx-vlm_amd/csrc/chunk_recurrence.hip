// Chunk-parallel form of the fixed-decay matrix-state recurrence of linear_recurrence.hip (no rotation):
//
//     S_t = a S_(t-1) + k_t v_t^T      o_t = S_t^T q_t          S: [D, Dv] per head, q / k / v optionally through silu
//
// for segments of more than max_len tokens (shorter ones stay with the token-by-token kernel).  A segment is cut into chunks of
// CH = 64 tokens counted from its first one; with S_0 the state a chunk starts from and i, j = 0 .. n - 1 its tokens
//
//     o_i = a^(i + 1) S_0^T q_i + sum_(j <= i) a^(i - j) (q_i . k_j) v_j        S_n = a^n S_0 + U,   U = sum_j a^(n - 1 - j) k_j v_j^T
//
//   chunk_update_kernel   U of every chunk, all chunks at once       -> workspace [chunk][H][D][Dv]
//   chunk_scan_kernel     the recurrence over chunks, one lane per state entry: the workspace's U becomes the chunk's S_0, the
//                         slot's state moves to the segment's end
//   chunk_output_kernel   o of every chunk, all chunks at once       -> raw [token][H][Dv] fp32
// All products run on the fp32 matrix cores (v_mfma_f32_16x16x4_f32: fp32 operands, products and sums), straight from global memory
// into the operand layout - a lane's rows / columns of a tile are consecutive in memory, so the loads are 8 to 32 bytes wide and
// neither kernel needs LDS or a barrier.  In the output kernel the scores come out as S^T = K Q^T, keys 4 g + r of a tile in register
// r of lane group g, which is the operand layout of the product with V when step r contracts the keys 4 g + r.
// Chunks are numbered over all long segments of the step; a launch covers the chunks [c0, c0 + nc) the workspace has room for, and
// windows of chunks follow each other on the stream (the slot's state carries a segment from one window to the next).
#include "common.hpp"
#include "../../include/vlm_hip.h"
#include "recurrence_finish.hpp"
#include "chunk_recurrence.hpp"

namespace {

constexpr int CH = VLM_CHUNK;

__device__ __forceinline__ float silu_f(float x) { return x * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * x)); }

// a^n for n >= 0 (a >= 0), exact for n = 0 and a = 0
__device__ __forceinline__ float powi(float l2a, int n) { return n == 0 ? 1.f : __builtin_amdgcn_exp2f(l2a * (float)n); }

// N consecutive values of a row, the first `have` of which exist
template <int N> __device__ __forceinline__ void row_vals(const bf16_t* p, int have, bool vec, float* f) {
  if (vec && have >= N && N >= 4) {
#pragma unroll
    for (int i = 0; i < N / 4; ++i) {
      const uint2 a = reinterpret_cast<const uint2*>(p)[i];
      f[4 * i] = bf_lo(a.x); f[4 * i + 1] = bf_hi(a.x); f[4 * i + 2] = bf_lo(a.y); f[4 * i + 3] = bf_hi(a.y);
    }
  } else {
#pragma unroll
    for (int i = 0; i < N; ++i) f[i] = i < have ? bf2f(p[i]) : 0.f;
  }
}
template <int N> __device__ __forceinline__ void row_vals(const float* p, int have, bool vec, float* f) {
  if (vec && have >= N && N >= 4) {
#pragma unroll
    for (int i = 0; i < N / 4; ++i) {
      const float4 a = reinterpret_cast<const float4*>(p)[i];
      f[4 * i] = a.x; f[4 * i + 1] = a.y; f[4 * i + 2] = a.z; f[4 * i + 3] = a.w;
    }
  } else {
#pragma unroll
    for (int i = 0; i < N; ++i) f[i] = i < have ? p[i] : 0.f;
  }
}

// the segment and the first token of global chunk number c (false: the step has fewer chunks)
__device__ __forceinline__ bool find_chunk(const vlm_recurrence_args& p, int nseg, int max_len, int c, int& t0, int& n) {
  for (int s = 0; s < nseg; ++s) {
    const int b = p.seg_start[s], len = p.seg_start[s + 1] - b;
    if (len <= max_len) continue;
    const int k = (len + CH - 1) / CH;
    if (c < k) {
      t0 = b + c * CH;
      n = min(CH, len - c * CH);
      return true;
    }
    c -= k;
  }
  return false;
}

// grid (chunks, H, ceil(super tiles / 4)), 4 waves: a wave owns 64 x 64 entries of U.  Row block rb of the super tile holds rows
// 4 r16 + rb, so one load of four consecutive values feeds four row blocks (columns alike)
template <typename T>
__global__ __launch_bounds__(256) void chunk_update_kernel(vlm_recurrence_args p, int nseg, int max_len, int c0, float* __restrict__ ws) {
  const int h = blockIdx.y, lane = threadIdx.x & 63, r16 = lane & 15, g = lane >> 4, D = p.D, Dv = p.Dv;
  const int st = blockIdx.z * 4 + (threadIdx.x >> 6), sc = (Dv + 63) / 64;
  if (st >= ((D + 63) / 64) * sc) return;
  int t0, n;
  if (!find_chunk(p, nseg, max_len, c0 + blockIdx.x, t0, n)) return;
  const int d0 = (st / sc) * 64 + 4 * r16, v0 = (st % sc) * 64 + 4 * r16;
  const T* k = (const T*)p.k + (long)h * D + d0;
  const T* v = (const T*)p.v + (long)h * Dv + v0;
  const bool kvec = ((uintptr_t)p.k % (4 * sizeof(T))) == 0 && p.ldk % 4 == 0 && D % 4 == 0;
  const bool vvec = ((uintptr_t)p.v % (4 * sizeof(T))) == 0 && p.ldv % 4 == 0 && Dv % 4 == 0;
  const float l2a = __builtin_amdgcn_logf(p.decay[h]);                   // log2
  f32x4_t acc[4][4];
#pragma unroll
  for (int a = 0; a < 4; ++a)
#pragma unroll
    for (int b = 0; b < 4; ++b) acc[a][b] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
  for (int j0 = 0; j0 < n; j0 += 4) {
    const int j = j0 + g;
    const bool live = j < n;
    const long tok = t0 + (live ? j : 0);
    float kv[4], vv[4];
    row_vals<4>(k + tok * p.ldk, live ? D - d0 : 0, kvec, kv);
    row_vals<4>(v + tok * p.ldv, live ? Dv - v0 : 0, vvec, vv);
    const float w = live ? powi(l2a, n - 1 - j) * p.kscale : 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      kv[i] = (p.k_act ? silu_f(kv[i]) : kv[i]) * w;
      vv[i] = p.v_act ? silu_f(vv[i]) : vv[i];
    }
#pragma unroll
    for (int a = 0; a < 4; ++a)
#pragma unroll
      for (int b = 0; b < 4; ++b) acc[a][b] = __builtin_amdgcn_mfma_f32_16x16x4f32(kv[a], vv[b], acc[a][b], 0, 0, 0);
  }
  // tile (a, b): row 4 (4 g + r) + a, column 4 r16 + b of the super tile
  float* U = ws + ((long)blockIdx.x * p.H + h) * (long)D * Dv;
#pragma unroll
  for (int a = 0; a < 4; ++a)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = (st / sc) * 64 + 4 * (4 * g + r) + a;
      if (d >= D) continue;
      float* u = U + (long)d * Dv + v0;
      if (Dv % 4 == 0) {
        if (v0 < Dv) *reinterpret_cast<float4*>(u) = make_float4(acc[a][0][r], acc[a][1][r], acc[a][2][r], acc[a][3][r]);
      } else {
#pragma unroll
        for (int b = 0; b < 4; ++b)
          if (v0 + b < Dv) u[b] = acc[a][b][r];
      }
    }
}

// grid (state entries / 256, nseg)
__global__ __launch_bounds__(256) void chunk_scan_kernel(vlm_recurrence_args p, int nseg, int max_len, int c0, int nc, float* __restrict__ ws) {
  const int seg = blockIdx.y;
  const int b = p.seg_start[seg], len = p.seg_start[seg + 1] - b;
  if (len <= max_len) return;
  int before = 0;                                                        // chunks of the long segments ahead of this one
  for (int s = 0; s < seg; ++s) {
    const int l = p.seg_start[s + 1] - p.seg_start[s];
    if (l > max_len) before += (l + CH - 1) / CH;
  }
  const int chunks = (len + CH - 1) / CH;
  const int lo = max(0, c0 - before), hi = min(chunks, c0 + nc - before);  // the segment's chunks inside the window
  if (lo >= hi) return;
  const long E = (long)p.D * p.Dv, HE = (long)p.H * E, e = (long)blockIdx.x * 256 + threadIdx.x;
  if (e >= HE) return;
  const float a = p.decay[e / E], l2a = __builtin_amdgcn_logf(a);
  float* S = p.state + (long)p.seg_slot[seg] * HE + e;
  float s = (lo > 0 || p.seg_pos0[seg] > 0) ? *S : 0.f;
  const float full = powi(l2a, CH);
  float* w = ws + (long)(before + lo - c0) * HE + e;
  int c = lo;
  for (; c + 4 < hi; c += 4, w += 4 * HE) {                              // whole chunks, four loads in flight
    float u[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) u[i] = w[i * HE];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      w[i * HE] = s;
      s = fmaf(full, s, u[i]);
    }
  }
  for (; c < hi; ++c, w += HE) {
    const float u = *w;
    *w = s;
    s = fmaf(c + 1 < chunks ? full : powi(l2a, len - c * CH), s, u);
  }
  *S = s;
}

// grid (chunks, H, value column tiles of 16 NB), 4 waves: wave w owns tokens 16 w .. 16 w + 15 of the chunk
template <typename T, int NB>
__global__ __launch_bounds__(256) void chunk_output_kernel(vlm_recurrence_args p, int nseg, int max_len, int c0, const float* __restrict__ ws) {
  const int h = blockIdx.y, wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r16 = lane & 15, g = lane >> 4, D = p.D, Dv = p.Dv;
  int t0, n;
  if (!find_chunk(p, nseg, max_len, c0 + blockIdx.x, t0, n)) return;
  const int i = wave * 16 + r16;                                         // this lane's query
  if (wave * 16 >= n) return;
  const int vcol = blockIdx.z * 16 * NB + r16 * NB, vhave = Dv - vcol;
  const T* qp = (const T*)p.q + (long)(t0 + min(i, n - 1)) * p.ldq + (long)h * D;
  const T* kp = (const T*)p.k + (long)t0 * p.ldk + (long)h * D;
  const T* vp = (const T*)p.v + (long)t0 * p.ldv + (long)h * Dv + vcol;
  const bool qvec = ((uintptr_t)p.q % (4 * sizeof(T))) == 0 && p.ldq % 4 == 0 && D % 4 == 0;
  const bool kvec = ((uintptr_t)p.k % (4 * sizeof(T))) == 0 && p.ldk % 4 == 0 && D % 4 == 0;
  const bool vvec = ((uintptr_t)p.v % (4 * sizeof(T))) == 0 && p.ldv % 4 == 0 && Dv % 4 == 0;
  const float* S = ws + ((long)blockIdx.x * p.H + h) * (long)D * Dv + vcol;
  const bool svec = Dv % 4 == 0;
  const float l2a = __builtin_amdgcn_logf(p.decay[h]);
  f32x4_t acc[NB], s[4];
#pragma unroll
  for (int b = 0; b < NB; ++b) acc[b] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int t = 0; t < 4; ++t) s[t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int c = 0; c < D; c += 16) {
    const int d = c + 4 * g;
    float q[4];
    row_vals<4>(qp + d, D - d, qvec, q);
#pragma unroll
    for (int x = 0; x < 4; ++x) q[x] = (p.q_act ? silu_f(q[x]) : q[x]) * p.qscale;
    // scores against the key tiles up to the wave's own
#pragma unroll
    for (int t = 0; t < 4; ++t) {
      if (t > wave) break;
      float k[4];
      row_vals<4>(kp + (long)min(t * 16 + r16, n - 1) * p.ldk + d, D - d, kvec, k);
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        k[x] = (p.k_act ? silu_f(k[x]) : k[x]) * p.kscale;
        s[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(k[x], q[x], s[t], 0, 0, 0);
      }
    }
    // the state the chunk starts from
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      float sv[NB];
      row_vals<NB>(S + (long)min(d + x, D - 1) * Dv, d + x < D ? vhave : 0, svec, sv);
#pragma unroll
      for (int b = 0; b < NB; ++b) acc[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(sv[b], q[x], acc[b], 0, 0, 0);
    }
  }
  const float ai = powi(l2a, i + 1);
#pragma unroll
  for (int b = 0; b < NB; ++b) acc[b] *= ai;
#pragma unroll
  for (int t = 0; t < 4; ++t) {
    if (t > wave) break;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int j = t * 16 + 4 * g + r;
      const float pr = j <= i ? s[t][r] * powi(l2a, i - j) : 0.f;        // (tokens past the chunk's end are later than every real query)
      float v[NB];
      row_vals<NB>(vp + (long)min(j, n - 1) * p.ldv, vhave, vvec, v);
#pragma unroll
      for (int b = 0; b < NB; ++b) acc[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(p.v_act ? silu_f(v[b]) : v[b], pr, acc[b], 0, 0, 0);
    }
  }
  if (i >= n) return;
  // block b, register r of lane group g: column (4 g + r) NB + b of the tile
  float* o = p.raw + ((long)(t0 + i) * p.H + h) * Dv;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int c = blockIdx.z * 16 * NB + (4 * g + r) * NB;
    if (NB % 4 == 0 && Dv % 4 == 0) {
#pragma unroll
      for (int b = 0; b < NB; b += 4)
        if (c + b < Dv) *reinterpret_cast<float4*>(o + c + b) = make_float4(acc[b][r], acc[(b + 1) % NB][r], acc[(b + 2) % NB][r], acc[(b + 3) % NB][r]);
    } else {
#pragma unroll
      for (int b = 0; b < NB; ++b)
        if (c + b < Dv) o[c + b] = acc[b][r];
    }
  }
}

template <typename T>
int run_chunks(const vlm_recurrence_args& a, int nseg, int ntok, int max_len, hipStream_t st) {
  const long HE = (long)a.H * a.D * a.Dv;
  const int total = ntok / CH + nseg;                                    // at most this many chunks
  const long room = a.ws_floats / HE;
  if (room < 1) return VLM_ERR_ARG;
  const int win = (int)(room < total ? room : total);
  const int tiles = ((a.D + 63) / 64) * ((a.Dv + 63) / 64);
  const int NB = a.Dv <= 16 ? 1 : a.Dv <= 64 ? 4 : 8, vt = (a.Dv + 16 * NB - 1) / (16 * NB);
  if ((HE + 255) / 256 > 0x7fffffffL || nseg > 65535) return VLM_ERR_SHAPE;
  for (int c0 = 0; c0 < total; c0 += win) {
    const int nc = total - c0 < win ? total - c0 : win;
    hipLaunchKernelGGL(chunk_update_kernel<T>, dim3(nc, a.H, (tiles + 3) / 4), dim3(256), 0, st, a, nseg, max_len, c0, a.ws);
    VLM_CHECK_LAUNCH();
    hipLaunchKernelGGL(chunk_scan_kernel, dim3((unsigned)((HE + 255) / 256), nseg), dim3(256), 0, st, a, nseg, max_len, c0, nc, a.ws);
    VLM_CHECK_LAUNCH();
    const dim3 grid(nc, a.H, vt);
    if (NB == 1) hipLaunchKernelGGL((chunk_output_kernel<T, 1>), grid, dim3(256), 0, st, a, nseg, max_len, c0, a.ws);
    else if (NB == 4) hipLaunchKernelGGL((chunk_output_kernel<T, 4>), grid, dim3(256), 0, st, a, nseg, max_len, c0, a.ws);
    else hipLaunchKernelGGL((chunk_output_kernel<T, 8>), grid, dim3(256), 0, st, a, nseg, max_len, c0, a.ws);
    VLM_CHECK_LAUNCH();
  }
  return VLM_OK;
}

}  // namespace

int vlm_chunk_recurrence(const vlm_recurrence_args* a, int nseg, int ntok, int max_len, int dtype, hipStream_t st) {
  return dtype ? run_chunks<float>(*a, nseg, ntok, max_len, st) : run_chunks<bf16_t>(*a, nseg, ntok, max_len, st);
}
