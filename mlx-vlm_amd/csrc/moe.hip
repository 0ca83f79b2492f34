// Mixture-of-experts routing and the expert activation, for experts whose up / down projections are stacked into ONE matrix
// each (rows of W_up: expert 0's ff rows, expert 1's, ..., then the shared expert's; columns of W_down in the same order).
// A token's routed output is then   down( gate_e(t) * act(up_e h) for every expert e )   with gate_e(t) = 0 for the experts
// the token did not choose: one up GEMM, this activation pass, one down GEMM - the sum over experts is the k loop of the down
// projection, and the experts a token skipped contribute exact zeros.
//
//   vlm_moe_route        logits fp32 [T][E] -> the `top` largest per token (lowest index wins a tie), softmax over the chosen
//                        logits only; dense gate table fp32 [T][E] (0 where not chosen) + the chosen (index, weight) lists
//   vlm_moe_route_scored the same choice with the weights taken from the softmax over ALL experts, times `scale`, with no
//                        second normalisation over the chosen ones; and group-limited: consecutive experts are cut into
//                        `groups` blocks of one size, a block ranks by its best expert, and the choice is made among the
//                        experts of the `keep` top-ranked blocks (lowest index wins a tie).  groups = keep = 1: no limit.
//   vlm_moe_route_sigmoid  scores s = sigmoid(z) per expert; the choice is made on s + correction (a per-expert offset that enters
//                        nothing but the choice), limited to the `keep` best blocks of experts, a block ranking by the SUM of its
//                        `group_top` largest choice scores; the experts of the other blocks cannot be chosen whatever their
//                        scores (not even when the kept ones are negative); weights = the chosen s, divided by their sum + 1e-20
//                        (when normalise), times scale.  The sigmoid of `extra` further logit columns is handed out beside the
//                        table: the gate of an expert that every token uses.
//   vlm_moe_router_softmax  router logits AND choice in one kernel: z = W_r h (fp32 sums), scores s = softmax(z) over all E columns, the
//                        `top` largest of s + correction (an offset per column that enters nothing but the choice; lowest index wins a
//                        tie) keep the weight s, not renormalised.  The last `identity` columns stand for experts that hand their
//                        input on: they have no column in the gate table [T][E - identity], the sum of their weights is handed
//                        out per token.
//   vlm_glu_rows         out[t][c] = act(g[t][c]) * u[t][c]; act: 0 = tanh-form gelu, 1 = silu, 2 = sigmoid, 4 = relu, 3 = clamped
//                        gate: with g' = min(g, limit), u' = clamp(u, -limit, limit): g' sigmoid(1.702 g') (u' + 1).  With a route table:
//                        E stacked experts of ff output columns, out[t][e ff + j] = act(g[t][e estride + j]) * u[t][e estride + j]
//                        * route[t][e] (estride: the distance of two experts' columns in g and u, e.g. 2 ff when every expert's
//                        gate and up rows lie side by side); without a route table g and u can get biases first; T-typed in and
//                        out, fp32 inside
//   vlm_moe_relu2_gate   out[t][c] = relu(up[t][c])^2 * gate[t][c / ff]   for c < E * ff,   relu(up[t][c])^2 for the
//                        `shared` columns behind them (an expert every token uses); T-typed in and out, fp32 inside
#include "common.hpp"
#include "../../include/vlm_hip.h"

namespace {

template <typename T> __device__ __forceinline__ float ld_f(const T* p);
template <> __device__ __forceinline__ float ld_f<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ld_f<bf16_t>(const bf16_t* p) { return bf2f(*p); }
template <typename T> __device__ __forceinline__ void st_f(T* p, float v);
template <> __device__ __forceinline__ void st_f<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void st_f<bf16_t>(bf16_t* p, float v) { *p = f2bf(v); }

// one wave per token; lane l owns experts l, l + 64, ... (a bit per owned expert records what earlier rounds took)
// scored: weights = softmax over all experts * scale (else: softmax over the chosen logits); groups / keep: see the file head
__global__ __launch_bounds__(256) void moe_route_kernel(const float* __restrict__ z, int T, int E, int top, int scored, int groups,
                                                        int keep, float scale, float* __restrict__ gate, int* __restrict__ idx,
                                                        float* __restrict__ wgt) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (t >= T) return;
  const float* zr = z + (long)t * E;
  for (int e = lane; e < E; e += 64) gate[(long)t * E + e] = 0.f;
  unsigned taken = 0u;                   // bit i: the lane's i-th expert is chosen, or (set before the choice) not eligible
  float all_max = 0.f, all_den = 1.f;
  if (scored) {                          // maximum and denominator over ALL experts, fixed order: lane-strided, then the xor tree
    float m = -INFINITY;
    for (int e = lane; e < E; e += 64) m = fmaxf(m, zr[e]);
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) m = fmaxf(m, __shfl_xor(m, o));
    float d = 0.f;
    for (int e = lane; e < E; e += 64) d += expf(zr[e] - m);
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) d += __shfl_xor(d, o);
    all_max = m;
    all_den = d;
  }
  if (groups > 1 && keep < groups) {     // rank the blocks by their best expert, keep `keep` of them; the experts of every other block are marked
    const int gsz = E / groups;
    unsigned long long kept = 0ull;      // (groups <= 64)
    for (int k = 0; k < keep; ++k) {
      float best = -INFINITY;
      int bg = 0x7fffffff;
      for (int e = lane; e < E; e += 64) {
        const int g = e / gsz;
        const float v = zr[e];
        if (!((kept >> g) & 1ull) && (v > best || (v == best && g < bg))) {
          best = v;
          bg = g;
        }
      }
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) {
        const float ob = __shfl_xor(best, o);
        const int og = __shfl_xor(bg, o);
        if (ob > best || (ob == best && og < bg)) {
          best = ob;
          bg = og;
        }
      }
      if (bg == 0x7fffffff) break;
      kept |= 1ull << bg;
    }
    for (int e = lane, i = 0; e < E; e += 64, ++i)
      if (!((kept >> (e / gsz)) & 1ull)) taken |= 1u << i;
  }
  float zmax = 0.f, denom = 0.f;
  float my_val = 0.f;                    // lane j < top keeps the j-th chosen logit
  int my_idx = -1;
  for (int j = 0; j < top; ++j) {
    float best = -INFINITY;
    int bi = 0x7fffffff;
    for (int e = lane, i = 0; e < E; e += 64, ++i) {
      const float v = zr[e];
      if (!((taken >> i) & 1u) && (v > best || (v == best && e < bi))) {
        best = v;
        bi = e;
      }
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ob = __shfl_xor(best, o);
      const int oi = __shfl_xor(bi, o);
      if (ob > best || (ob == best && oi < bi)) {
        best = ob;
        bi = oi;
      }
    }
    if (bi == 0x7fffffff) break;         // fewer comparable candidates than `top` (NaN logits): what was found is kept
    if (lane == (bi & 63)) taken |= 1u << (bi >> 6);
    if (j == 0) zmax = best;
    if (lane == j) {
      my_val = best;
      my_idx = bi;
    }
    denom += expf(best - zmax);
  }
  const float w = my_idx < 0 ? 0.f : (scored ? expf(my_val - all_max) / all_den * scale : expf(my_val - zmax) / denom);
  if (lane < top) {
    idx[(long)t * top + lane] = my_idx < 0 ? 0 : my_idx;
    wgt[(long)t * top + lane] = w;
  }
  for (int j = 0; j < top; ++j) {        // the owner of an expert writes its gate (it also wrote the zero)
    const int ej = __shfl(my_idx, j);
    const float wj = __shfl(w, j);
    if (ej >= 0 && lane == (ej & 63)) gate[(long)t * E + ej] = wj;
  }
}

// one wave per token; lane l owns experts l, l + 64, ... (bit i of `taken`: the lane's i-th expert is chosen or not eligible)
__global__ __launch_bounds__(256) void moe_route_sigmoid_kernel(const float* __restrict__ z, long ldz, int T, int E, int top, int groups,
                                                                int keep, int group_top, const float* __restrict__ corr, int normalise,
                                                                float scale, int extra, float* __restrict__ extra_out,
                                                                float* __restrict__ gate, int* __restrict__ idx, float* __restrict__ wgt) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (t >= T) return;
  const float* zr = z + (long)t * ldz;
  for (int e = lane; e < E; e += 64) gate[(long)t * E + e] = 0.f;
  for (int e = lane; e < extra; e += 64) extra_out[(long)t * extra + e] = 1.f / (1.f + expf(-zr[E + e]));
  auto choice = [&](int e) { return 1.f / (1.f + expf(-zr[e])) + (corr ? corr[e] : 0.f); };
  unsigned taken = 0u;
  if (groups > 1 && keep < groups) {
    const int gsz = E / groups;
    // lane g (groups <= 64): the sum of the group_top largest choice scores of block g, members taken in index order
    float gscore = -INFINITY;
    if (lane < groups) {
      float sum = 0.f;
      int last = -1;
      float lastv = INFINITY;
      for (int k = 0; k < group_top && k < gsz; ++k) {   // k-th largest: the largest value below (lastv, last) in (value desc, index asc) order
        float best = -INFINITY;
        int bi = -1;
        for (int j = 0; j < gsz; ++j) {
          const float v = choice(lane * gsz + j);
          const bool below = v < lastv || (v == lastv && j > last);
          if (below && (bi < 0 || v > best)) {
            best = v;
            bi = j;
          }
        }
        if (bi < 0) break;
        sum += best;
        lastv = best;
        last = bi;
      }
      gscore = sum;
    }
    unsigned long long kept = 0ull;
    for (int k = 0; k < keep; ++k) {
      float best = (lane < groups && !((kept >> lane) & 1ull)) ? gscore : -INFINITY;
      int bg = (lane < groups && !((kept >> lane) & 1ull)) ? lane : 0x7fffffff;
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) {
        const float ob = __shfl_xor(best, o);
        const int og = __shfl_xor(bg, o);
        if (og != 0x7fffffff && (bg == 0x7fffffff || ob > best || (ob == best && og < bg))) {
          best = ob;
          bg = og;
        }
      }
      if (bg == 0x7fffffff) break;
      kept |= 1ull << bg;
    }
    for (int e = lane, i = 0; e < E; e += 64, ++i)
      if (!((kept >> (e / gsz)) & 1ull)) taken |= 1u << i;
  }
  float my_s = 0.f, denom = 0.f;
  int my_idx = -1;
  for (int j = 0; j < top; ++j) {
    float best = -INFINITY;
    int bi = 0x7fffffff;
    for (int e = lane, i = 0; e < E; e += 64, ++i) {
      if ((taken >> i) & 1u) continue;
      const float v = choice(e);
      if (bi == 0x7fffffff || v > best || (v == best && e < bi)) {
        best = v;
        bi = e;
      }
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ob = __shfl_xor(best, o);
      const int oi = __shfl_xor(bi, o);
      if (oi != 0x7fffffff && (bi == 0x7fffffff || ob > best || (ob == best && oi < bi))) {
        best = ob;
        bi = oi;
      }
    }
    if (bi == 0x7fffffff) break;
    if (lane == (bi & 63)) taken |= 1u << (bi >> 6);
    const float sj = 1.f / (1.f + expf(-zr[bi]));        // the weight uses the score WITHOUT the correction
    if (lane == j) {
      my_s = sj;
      my_idx = bi;
    }
    denom += sj;                                         // chosen order, the same in every lane
  }
  const float w = my_idx < 0 ? 0.f : (normalise ? my_s / (denom + 1e-20f) : my_s) * scale;
  if (lane < top) {
    idx[(long)t * top + lane] = my_idx < 0 ? 0 : my_idx;
    wgt[(long)t * top + lane] = w;
  }
  for (int j = 0; j < top; ++j) {
    const int ej = __shfl(my_idx, j);
    const float wj = __shfl(w, j);
    if (ej >= 0 && lane == (ej & 63)) gate[(long)t * E + ej] = wj;
  }
}

// Workgroup = 16 tokens.  Logits: bf16 rows of whole 16-byte pieces (MFMA) on v_mfma_f32_16x16x32_bf16, 16 experts x 16 tokens per product,
// the waves share the k steps and add their partial sums in wave order; else one token per wave and expert, lanes over k.  Then one
// wave per 4 tokens chooses: lane l owns the experts l + 64 i.
template <typename T, int EG, bool MFMA>
__global__ __launch_bounds__(256) void moe_router_softmax_kernel(const T* __restrict__ h, long ldh, const T* __restrict__ w, long ldw, int D,
                                                                 int rows, int E, int top, int identity, const float* __restrict__ corr,
                                                                 float* __restrict__ gate, float* __restrict__ ident) {
  typedef __attribute__((ext_vector_type(8))) __bf16 bf8;
  __shared__ float z[16][EG * 16 + 1];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, t0 = blockIdx.x * 16;
  if constexpr (MFMA) {
    const int r16 = lane & 15, g = lane >> 4;
    f32x4_t acc[EG];
#pragma unroll
    for (int e = 0; e < EG; ++e) acc[e] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const T* hr = h + (long)min(t0 + r16, rows - 1) * ldh;
#pragma unroll 2
    for (int c = wave * 32; c < D; c += 128) {
      const int d = c + 8 * g;
      const u32x4_t none = {0u, 0u, 0u, 0u};
      bf8 b = __builtin_bit_cast(bf8, none);
      if (d < D) b = *reinterpret_cast<const bf8*>(hr + d);
#pragma unroll
      for (int e = 0; e < EG; ++e) {
        bf8 a = __builtin_bit_cast(bf8, none);
        if (d < D) a = *reinterpret_cast<const bf8*>(w + (long)min(e * 16 + r16, E - 1) * ldw + d);
        acc[e] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, acc[e], 0, 0, 0);
      }
    }
    for (int k = 0; k < 4; ++k) {
      if (wave == k) {
#pragma unroll
        for (int e = 0; e < EG; ++e)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            float* p = &z[r16][e * 16 + 4 * g + r];
            *p = k == 0 ? acc[e][r] : *p + acc[e][r];
          }
      }
      __syncthreads();
    }
  } else {
    for (int j = 0; j < 4; ++j) {
      const int t = t0 + wave * 4 + j;
      if (t >= rows) break;
      for (int e = 0; e < E; ++e) {
        float s = 0.f;
        for (int d = lane; d < D; d += 64) s = fmaf(ld_f(h + (long)t * ldh + d), ld_f(w + (long)e * ldw + d), s);
        s = wave_sum(s);
        if (lane == 0) z[wave * 4 + j][e] = s;
      }
    }
    __syncthreads();
  }
  constexpr int NI = (EG * 16 + 63) / 64;                // experts per lane
  const int Er = E - identity;
  for (int j = 0; j < 4; ++j) {
    const int t = t0 + wave * 4 + j;
    if (t >= rows) break;                                // (uniform over the wave)
    const float* zr = z[wave * 4 + j];
    float s[NI], c[NI], m = -INFINITY;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int e = lane + 64 * i;
      s[i] = e < E ? zr[e] : -INFINITY;
      m = fmaxf(m, s[i]);
    }
    m = wave_max(m);
    float den = 0.f;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      s[i] = lane + 64 * i < E ? expf(s[i] - m) : 0.f;
      den += s[i];
    }
    den = wave_sum(den);
    float keep[NI];
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int e = lane + 64 * i;
      s[i] /= den;
      c[i] = e < E ? s[i] + (corr ? corr[e] : 0.f) : -INFINITY;
      keep[i] = 0.f;
    }
    unsigned taken = 0u;
    for (int k = 0; k < top; ++k) {
      float best = -INFINITY;
      int bi = 0x7fffffff;
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        const int e = lane + 64 * i;
        if (e < E && !((taken >> i) & 1u) && (bi == 0x7fffffff || c[i] > best)) {
          best = c[i];
          bi = e;
        }
      }
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) {
        const float ob = __shfl_xor(best, o);
        const int oi = __shfl_xor(bi, o);
        if (oi != 0x7fffffff && (bi == 0x7fffffff || ob > best || (ob == best && oi < bi))) {
          best = ob;
          bi = oi;
        }
      }
      if (bi == 0x7fffffff) break;
      if (lane == (bi & 63)) {
        taken |= 1u << (bi >> 6);
#pragma unroll
        for (int i = 0; i < NI; ++i)
          if (i == bi >> 6) keep[i] = s[i];
      }
    }
    float id = 0.f;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int e = lane + 64 * i;
      if (e < Er) gate[(long)t * Er + e] = keep[i];
      else id += keep[i];
    }
    if (identity) {
      id = wave_sum(id);
      if (lane == 0) ident[t] = id;
    }
  }
}

template <typename T>
__global__ __launch_bounds__(256) void moe_relu2_gate_kernel(const T* __restrict__ up, long ldu, const float* __restrict__ gate, int E,
                                                             int ff, int shared, T* __restrict__ out, long ldo, int rows) {
  const int cols = E * ff + shared;
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= (long)rows * cols) return;
  const long t = i / cols;
  const int c = (int)(i % cols);
  const float u = fmaxf(ld_f(up + t * ldu + c), 0.f);
  const float g = c < E * ff ? gate[t * E + c / ff] : 1.f;
  st_f(out + t * ldo + c, u * u * g);
}

__device__ __forceinline__ float glu_act(float z, int act) {
  if (act == 4) return fmaxf(z, 0.f);
  if (act == 0) return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
  const float sg = 1.f / (1.f + expf(-z));
  return act == 1 ? z * sg : sg;
}

__device__ __forceinline__ float clamped_glu(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g / (1.f + expf(-1.702f * g)) * (u + 1.f);
}

template <typename T>
__global__ __launch_bounds__(256) void glu_rows_kernel(const T* __restrict__ g, long ldg, const T* __restrict__ u, long ldu,
                                                       const float* __restrict__ route, int E, int ff, int estride, int act,
                                                       float limit, const T* __restrict__ gb, const T* __restrict__ ub, T* __restrict__ out, long ldo, int rows,
                                                       int dim) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= (long)rows * dim) return;
  const long t = i / dim;
  const int c = (int)(i % dim);
  float r = 1.f;
  long cs = c;                            // the column in g and u
  if (route) {
    const int e = c / ff;
    r = route[t * E + e];
    if (r == 0.f) {                       // an expert the token did not choose: an exact zero whatever its columns hold
      st_f(out + t * ldo + c, 0.f);
      return;
    }
    cs = (long)e * estride + (c - e * ff);
  }
  const float gv = ld_f(g + t * ldg + cs) + (gb ? ld_f(gb + c) : 0.f), uv = ld_f(u + t * ldu + cs) + (ub ? ld_f(ub + c) : 0.f);
  st_f(out + t * ldo + c, (act == 3 ? clamped_glu(gv, uv, limit) : glu_act(gv, act) * uv) * r);
}

// bf16 rows whose columns come in whole groups of 8 (16-byte accesses), for the clamped gate (act 3, optionally over stacked experts with a
// route table, ff a multiple of 8) and relu (act 4, optionally with biases)
__device__ __forceinline__ void load8f(const bf16_t* p, float* f) {
  const uint4 v = *reinterpret_cast<const uint4*>(p);
  f[0] = bf_lo(v.x); f[1] = bf_hi(v.x); f[2] = bf_lo(v.y); f[3] = bf_hi(v.y);
  f[4] = bf_lo(v.z); f[5] = bf_hi(v.z); f[6] = bf_lo(v.w); f[7] = bf_hi(v.w);
}
template <int ACT, bool ROUTE>
__global__ __launch_bounds__(256) void glu_vec_kernel(const bf16_t* __restrict__ g, long ldg, const bf16_t* __restrict__ u, long ldu,
                                                      const float* __restrict__ route, int E, int ff, int estride, float limit,
                                                      const bf16_t* __restrict__ gb, const bf16_t* __restrict__ ub,
                                                      bf16_t* __restrict__ out, long ldo, int rows, int dim8) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= (long)rows * dim8) return;
  const long t = i / dim8;
  const int c = (int)(i % dim8) * 8;
  long cs = c;
  float r = 1.f;
  if constexpr (ROUTE) {
    const int e = c / ff;
    r = route[t * E + e];
    if (r == 0.f) {
      *reinterpret_cast<uint4*>(out + t * ldo + c) = make_uint4(0u, 0u, 0u, 0u);
      return;
    }
    cs = (long)e * estride + (c - e * ff);
  }
  float gv[8], uv[8];
  load8f(g + t * ldg + cs, gv);
  load8f(u + t * ldu + cs, uv);
  if (ACT == 4 && gb) {
#pragma unroll
    for (int j = 0; j < 8; ++j) gv[j] += bf2f(gb[c + j]);
  }
  if (ACT == 4 && ub) {
#pragma unroll
    for (int j = 0; j < 8; ++j) uv[j] += bf2f(ub[c + j]);
  }
  float v[8];
#pragma unroll
  for (int j = 0; j < 8; ++j) v[j] = ACT == 3 ? clamped_glu(gv[j], uv[j], limit) * r : fmaxf(gv[j], 0.f) * uv[j];
  *reinterpret_cast<uint4*>(out + t * ldo + c) = make_uint4(pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3]), pack_bf2(v[4], v[5]), pack_bf2(v[6], v[7]));
}

}  // namespace

extern "C" int vlm_moe_route(const void* logits, int T, int E, int top, void* gate, void* idx, void* wgt, void* stream) {
  if (!logits || !gate || !idx || !wgt || T < 0 || E <= 0 || top <= 0 || top > E) return VLM_ERR_ARG;
  if (top > 64 || E > 2048) return VLM_ERR_SHAPE;
  if (T == 0) return VLM_OK;
  hipLaunchKernelGGL(moe_route_kernel, dim3((T + 3) / 4), dim3(256), 0, (hipStream_t)stream, (const float*)logits, T, E, top, 0, 1, 1,
                     1.f, (float*)gate, (int*)idx, (float*)wgt);
  VLM_CHECK_LAUNCH();
  return VLM_OK;
}

extern "C" int vlm_moe_route_scored(const void* logits, int T, int E, int top, int groups, int keep, float scale, void* gate, void* idx,
                                    void* wgt, void* stream) {
  if (!logits || !gate || !idx || !wgt || T < 0 || E <= 0 || top <= 0 || top > E || groups <= 0 || keep <= 0 || keep > groups ||
      E % groups || top > (long)keep * (E / groups))
    return VLM_ERR_ARG;
  if (top > 64 || E > 2048 || groups > 64) return VLM_ERR_SHAPE;
  if (T == 0) return VLM_OK;
  hipLaunchKernelGGL(moe_route_kernel, dim3((T + 3) / 4), dim3(256), 0, (hipStream_t)stream, (const float*)logits, T, E, top, 1, groups,
                     keep, scale, (float*)gate, (int*)idx, (float*)wgt);
  VLM_CHECK_LAUNCH();
  return VLM_OK;
}

extern "C" int vlm_moe_route_sigmoid(const void* logits, long ldz, int T, int E, int top, int groups, int keep, int group_top,
                                     const void* correction, int normalise, float scale, int extra, void* extra_out, void* gate, void* idx,
                                     void* wgt, void* stream) {
  if (!logits || !gate || !idx || !wgt || T < 0 || E <= 0 || top <= 0 || top > E || groups <= 0 || keep <= 0 || keep > groups || E % groups ||
      top > (long)keep * (E / groups) || group_top < 1 || extra < 0 || (extra && !extra_out) || ldz < (long)E + extra)
    return VLM_ERR_ARG;
  if (top > 64 || E > 2048 || groups > 64) return VLM_ERR_SHAPE;
  if (T == 0) return VLM_OK;
  hipLaunchKernelGGL(moe_route_sigmoid_kernel, dim3((T + 3) / 4), dim3(256), 0, (hipStream_t)stream, (const float*)logits, ldz, T, E, top,
                     groups, keep, group_top, (const float*)correction, normalise, scale, extra, (float*)extra_out, (float*)gate, (int*)idx,
                     (float*)wgt);
  VLM_CHECK_LAUNCH();
  return VLM_OK;
}

extern "C" int vlm_moe_router_softmax(const void* h, long ldh, const void* w, long ldw, int D, int T, int E, int top, int identity,
                                      const void* correction, void* gate, void* ident, int dtype, void* stream) {
  if (!h || !w || D <= 0 || ldh < D || ldw < D || T < 0 || E <= 0 || top <= 0 || top > E || identity < 0 || identity > E ||
      (identity && !ident) || (identity < E && !gate))
    return VLM_ERR_ARG;
  if (E > 256) return VLM_ERR_SHAPE;
  if (T == 0) return VLM_OK;
  hipStream_t st = (hipStream_t)stream;
  const bool mfma = !dtype && D % 8 == 0 && ldh % 8 == 0 && ldw % 8 == 0 && (((uintptr_t)h | (uintptr_t)w) & 15) == 0;
#define GO(TT, EG, M)                                                                                                             \
  hipLaunchKernelGGL((moe_router_softmax_kernel<TT, EG, M>), dim3((T + 15) / 16), dim3(256), 0, st, (const TT*)h, ldh, (const TT*)w, ldw, D, T, E, \
                     top, identity, (const float*)correction, (float*)gate, (float*)ident)
#define GO2(EG) do { if (dtype) GO(float, EG, false); else if (mfma) GO(bf16_t, EG, true); else GO(bf16_t, EG, false); } while (0)
  if (E <= 16) GO2(1); else if (E <= 32) GO2(2); else if (E <= 64) GO2(4); else if (E <= 128) GO2(8); else GO2(16);
#undef GO2
#undef GO
  VLM_CHECK_LAUNCH();
  return VLM_OK;
}

extern "C" int vlm_glu_rows(const void* g, long ldg, const void* u, long ldu, const void* route, int E, int ff, int estride, int act,
                            float limit, const void* gbias, const void* ubias, void* out, long ldo, int rows, int dim, int dtype,
                            void* stream) {
  if (!g || !u || !out || rows < 0 || dim <= 0 || ldo < dim || act < 0 || act > 4 || (act == 3 && !(limit >= 0.f)) ||
      (route && (gbias || ubias)))
    return VLM_ERR_ARG;
  if (route ? (E <= 0 || ff <= 0 || (long)E * ff != dim || estride < ff || ldg < (long)(E - 1) * estride + ff ||
               ldu < (long)(E - 1) * estride + ff)
            : (ldg < dim || ldu < dim))
    return VLM_ERR_ARG;
  if (rows == 0) return VLM_OK;
  const unsigned nb = (unsigned)(((long)rows * dim + 255) / 256);
  hipStream_t st = (hipStream_t)stream;
  if (!dtype && (act == 3 ? !gbias && !ubias && (!route || (ff % 8 == 0 && estride % 8 == 0)) : act == 4 && !route) && dim % 8 == 0 &&
      ldg % 8 == 0 && ldu % 8 == 0 && ldo % 8 == 0 && (((uintptr_t)g | (uintptr_t)u | (uintptr_t)out) & 15) == 0) {
    const unsigned nv = (unsigned)(((long)rows * (dim / 8) + 255) / 256);
#define GO(A, R)                                                                                                                  \
  hipLaunchKernelGGL((glu_vec_kernel<A, R>), dim3(nv), dim3(256), 0, st, (const bf16_t*)g, ldg, (const bf16_t*)u, ldu, (const float*)route, E, ff, \
                     estride, limit, (const bf16_t*)gbias, (const bf16_t*)ubias, (bf16_t*)out, ldo, rows, dim / 8)
    if (act == 4) GO(4, false); else if (route) GO(3, true); else GO(3, false);
#undef GO
    VLM_CHECK_LAUNCH();
    return VLM_OK;
  }
#define GO(T)                                                                                                                     \
  hipLaunchKernelGGL(glu_rows_kernel<T>, dim3(nb), dim3(256), 0, st, (const T*)g, ldg, (const T*)u, ldu, (const float*)route, E, ff, estride, act, \
                     limit, (const T*)gbias, (const T*)ubias, (T*)out, ldo, rows, dim)
  if (dtype) GO(float); else GO(bf16_t);
#undef GO
  VLM_CHECK_LAUNCH();
  return VLM_OK;
}

extern "C" int vlm_moe_relu2_gate(const void* up, long ldu, const void* gate, int E, int ff, int shared, void* out, long ldo, int rows,
                                  int dtype, void* stream) {
  if (!up || !out || rows < 0 || E < 0 || ff < 0 || shared < 0 || (E > 0 && !gate)) return VLM_ERR_ARG;
  const long cols = (long)E * ff + shared;
  if (cols <= 0 || ldu < cols || ldo < cols) return VLM_ERR_ARG;
  if (rows == 0) return VLM_OK;
  const unsigned nb = (unsigned)((rows * cols + 255) / 256);
  hipStream_t st = (hipStream_t)stream;
  if (dtype)
    hipLaunchKernelGGL(moe_relu2_gate_kernel<float>, dim3(nb), dim3(256), 0, st, (const float*)up, ldu, (const float*)gate, E, ff,
                       shared, (float*)out, ldo, rows);
  else
    hipLaunchKernelGGL(moe_relu2_gate_kernel<bf16_t>, dim3(nb), dim3(256), 0, st, (const bf16_t*)up, ldu, (const float*)gate, E, ff,
                       shared, (bf16_t*)out, ldo, rows);
  VLM_CHECK_LAUNCH();
  return VLM_OK;
}
