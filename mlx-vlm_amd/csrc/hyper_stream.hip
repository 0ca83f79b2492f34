// Hyper-connections: the residual of a decoder as S fp32 streams per token that every sublayer reads through one weight per
// stream, and that are mixed with each other when its result is written back.  One pass per sublayer boundary:
//
//     write:  x'_t = sum_s mix[s][t] x_s + out[t] * y          (all new streams from the OLD ones; mix is indexed [from][to])
//     read:   u    = sum_t in[t] x'_t      h = u / sqrt(mean(u^2) + eps) * w       h: T-typed rows, the next sublayer's input
//
// Either half may be left out: without y the streams are only read, without `in` only written.  With S = 1 and weights of one
// this is the plain residual step.  Streams lie side by side per token, fp32 [tokens][S][D]; the source may also be ONE row per
// token that stands for all S streams (xin_stream = 0: the embedding rows before the first sublayer), so the copies never have
// to be made.  Reading all streams at once (every in[] one) gives their sum: the final norm.
//
//   vlm_hyper_step   workgroup = token; a lane owns the same columns of every stream, so the old streams stay in its registers
//                    while the new ones are formed and the update may run in place.  16-byte accesses when the pitches allow.
#include "common.hpp"
#include "../../include/vlm_hip.h"
#include "recurrence_finish.hpp"

namespace {

template <int V> struct fvec { float v[V]; };
template <int V> __device__ __forceinline__ fvec<V> ldv(const float* p);
template <> __device__ __forceinline__ fvec<1> ldv<1>(const float* p) { return {{*p}}; }
template <> __device__ __forceinline__ fvec<4> ldv<4>(const float* p) {
  const float4 a = *reinterpret_cast<const float4*>(p);
  return {{a.x, a.y, a.z, a.w}};
}
template <int V> __device__ __forceinline__ fvec<V> ldv(const bf16_t* p);
template <> __device__ __forceinline__ fvec<1> ldv<1>(const bf16_t* p) { return {{bf2f(*p)}}; }
template <> __device__ __forceinline__ fvec<4> ldv<4>(const bf16_t* p) {
  const uint2 a = *reinterpret_cast<const uint2*>(p);
  return {{bf_lo(a.x), bf_hi(a.x), bf_lo(a.y), bf_hi(a.y)}};
}
__device__ __forceinline__ void stv(float* p, const fvec<1>& f) { *p = f.v[0]; }
__device__ __forceinline__ void stv(float* p, const fvec<4>& f) { *reinterpret_cast<float4*>(p) = make_float4(f.v[0], f.v[1], f.v[2], f.v[3]); }
__device__ __forceinline__ void stv(bf16_t* p, const fvec<1>& f) { *p = f2bf(f.v[0]); }
__device__ __forceinline__ void stv(bf16_t* p, const fvec<4>& f) {
  *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf2(f.v[0], f.v[1]), pack_bf2(f.v[2], f.v[3]));
}

template <typename T, int S, int V>
__global__ __launch_bounds__(256) void hyper_step_kernel(vlm_hyper_args p) {
  extern __shared__ __align__(16) float us[];       // [D] the read-out before its norm
  __shared__ float red[4];
  const long t = blockIdx.x;
  const int D = p.D, tid = threadIdx.x, nthr = blockDim.x;
  const float* xin = p.xin + t * p.xin_tok;
  float* xo = p.xout ? p.xout + t * S * (long)D : nullptr;
  const T* y = p.y ? (const T*)p.y + t * p.ldy : nullptr;
  float cin[S], cout[S], mix[S * S];
#pragma unroll
  for (int s = 0; s < S; ++s) cin[s] = p.in ? p.in[s] : 1.f;
  if (y) {
#pragma unroll
    for (int s = 0; s < S; ++s) cout[s] = p.out[s];
#pragma unroll
    for (int s = 0; s < S * S; ++s) mix[s] = p.mix[s];
  }
  float q = 0.f;
  for (int d = tid * V; d < D; d += nthr * V) {
    fvec<V> x[S];
#pragma unroll
    for (int s = 0; s < S; ++s) x[s] = ldv<V>(xin + s * p.xin_stream + d);
    fvec<V> u;
#pragma unroll
    for (int i = 0; i < V; ++i) u.v[i] = 0.f;
    if (y) {
      const fvec<V> yv = ldv<V>(y + d);
#pragma unroll
      for (int to = 0; to < S; ++to) {
        fvec<V> n;
#pragma unroll
        for (int i = 0; i < V; ++i) {
          float a = cout[to] * yv.v[i];
#pragma unroll
          for (int s = 0; s < S; ++s) a = fmaf(mix[s * S + to], x[s].v[i], a);
          n.v[i] = a;
          u.v[i] = fmaf(cin[to], a, u.v[i]);
        }
        stv(xo + (long)to * D + d, n);
      }
    } else {
#pragma unroll
      for (int s = 0; s < S; ++s)
#pragma unroll
        for (int i = 0; i < V; ++i) u.v[i] = fmaf(cin[s], x[s].v[i], u.v[i]);
    }
    if (p.w) {
#pragma unroll
      for (int i = 0; i < V; ++i) {
        us[d + i] = u.v[i];                          // (every lane re-reads only the entries it wrote)
        q = fmaf(u.v[i], u.v[i], q);
      }
    }
  }
  if (!p.w) return;
  q = wave_sum(q);
  if ((tid & 63) == 0) red[tid >> 6] = q;
  __syncthreads();
  float tot = 0.f;
  for (int i = 0; i < nthr / 64; ++i) tot += red[i];
  const float r = 1.0f / sqrtf(tot / (float)D + p.eps);
  const T* w = (const T*)p.w;
  T* h = (T*)p.h + t * p.ldh;
  for (int d = tid * V; d < D; d += nthr * V) {
    const fvec<V> wv = ldv<V>(w + d);
    fvec<V> o;
#pragma unroll
    for (int i = 0; i < V; ++i) o.v[i] = us[d + i] * r * wv.v[i];
    stv(h + d, o);
  }
}

template <typename T, int S>
int launch(const vlm_hyper_args& a, int rows, hipStream_t st) {
  const size_t lds = a.w ? (size_t)a.D * sizeof(float) : 16;
  const int esz = sizeof(T);
  const bool vec = a.D % 4 == 0 && a.xin_tok % 4 == 0 && a.xin_stream % 4 == 0 && ((uintptr_t)a.xin & 15) == 0 && ((uintptr_t)a.xout & 15) == 0 &&
                   (!a.y || (a.ldy % 4 == 0 && ((uintptr_t)a.y & (4 * esz - 1)) == 0)) &&
                   (!a.w || (a.ldh % 4 == 0 && ((uintptr_t)a.h & (4 * esz - 1)) == 0 && ((uintptr_t)a.w & (4 * esz - 1)) == 0));
  if (vec) hipLaunchKernelGGL((hyper_step_kernel<T, S, 4>), dim3(rows), dim3(256), lds, st, a);
  else hipLaunchKernelGGL((hyper_step_kernel<T, S, 1>), dim3(rows), dim3(256), lds, st, a);
  VLM_CHECK_LAUNCH();
  return VLM_OK;
}

template <typename T>
int run(const vlm_hyper_args& a, int rows, hipStream_t st) {
  switch (a.S) {
    case 1: return launch<T, 1>(a, rows, st);
    case 2: return launch<T, 2>(a, rows, st);
    case 3: return launch<T, 3>(a, rows, st);
    case 4: return launch<T, 4>(a, rows, st);
    case 5: return launch<T, 5>(a, rows, st);
    case 6: return launch<T, 6>(a, rows, st);
    case 7: return launch<T, 7>(a, rows, st);
    case 8: return launch<T, 8>(a, rows, st);
    default: return VLM_ERR_SHAPE;
  }
}

}  // namespace

extern "C" int vlm_hyper_step(const vlm_hyper_args* a, int rows, int dtype, void* stream) {
  if (!a || !a->xin || a->S <= 0 || a->D <= 0 || rows < 0 || a->xin_tok < 0 || a->xin_stream < 0 || (!a->y && !a->w)) return VLM_ERR_ARG;
  if (a->xin_stream ? a->xin_tok < (long)(a->S - 1) * a->xin_stream + a->D : a->xin_tok < a->D) return VLM_ERR_ARG;
  if (a->y && (!a->xout || !a->mix || !a->out || a->ldy < a->D)) return VLM_ERR_ARG;
  if (a->w && (!a->h || a->ldh < a->D)) return VLM_ERR_ARG;
  if (a->S > 8 || a->D > 15360) return VLM_ERR_SHAPE;
  if (rows == 0) return VLM_OK;
  return dtype ? run<float>(*a, rows, (hipStream_t)stream) : run<bf16_t>(*a, rows, (hipStream_t)stream);
}
