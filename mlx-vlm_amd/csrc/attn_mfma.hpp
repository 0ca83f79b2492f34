// Shared by the matrix-core attentions over paged caches (diff_attn.hip, grouped_attn.hip, latent_attn_mfma.hip): loads of value
// columns in the layout the products take, operand pieces, and the split of fp32 values into two bf16 values.
//
// All of them work on transposed products: S^T = K Q^T leaves the scores of a query in one lane column, keys 4 g + r of a 16-key group in
// register r of lane group g, which is the operand layout of P^T in O^T += V^T P^T when the contraction runs over the keys in
// that order.
#pragma once
#include "common.hpp"

namespace {

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
typedef __attribute__((ext_vector_type(8))) __bf16 bf8;

__device__ __forceinline__ bf8 zero8() { return __builtin_bit_cast(bf8, u32x4_t{0u, 0u, 0u, 0u}); }

// value columns of one key as they are stored: NB fp32 values / NB bf16 values packed two to a register
template <typename T, int NB> struct VRow;
template <int NB> struct VRow<float, NB> {
  float f[NB];
  __device__ __forceinline__ void load(const float* p, int have, bool vec) { load_cols<NB>(p, have, vec, f); }
};
template <int NB> struct VRow<bf16_t, NB> {
  unsigned w[(NB + 1) / 2];
  __device__ __forceinline__ void load(const bf16_t* p, int have, bool vec) {
    if (vec && NB >= 8) {
#pragma unroll
      for (int i = 0; i < NB / 8; ++i) {
        uint4 a = make_uint4(0u, 0u, 0u, 0u);
        if (have > 0) a = reinterpret_cast<const uint4*>(p)[i];
        w[4 * i] = a.x; w[(4 * i + 1) % ((NB + 1) / 2)] = a.y; w[(4 * i + 2) % ((NB + 1) / 2)] = a.z; w[(4 * i + 3) % ((NB + 1) / 2)] = a.w;
      }
    } else if (vec && NB == 4) {
      uint2 a = make_uint2(0u, 0u);
      if (have > 0) a = *reinterpret_cast<const uint2*>(p);
      w[0] = a.x; w[1 % ((NB + 1) / 2)] = a.y;
    } else {
#pragma unroll
      for (int i = 0; i < (NB + 1) / 2; ++i)
        w[i] = (2 * i < have ? (unsigned)p[2 * i] : 0u) | (2 * i + 1 < NB && 2 * i + 1 < have ? (unsigned)p[2 * i + 1] << 16 : 0u);
    }
  }
};
// column b of two keys, the first in the low half
__device__ __forceinline__ unsigned pair_cols(unsigned a, unsigned b, int odd) {
  return odd ? __builtin_amdgcn_perm(b, a, 0x07060302u) : __builtin_amdgcn_perm(b, a, 0x05040100u);
}

// 8 fp32 values as hi + lo bf16 operands (contraction order: the values' own)
__device__ __forceinline__ void split8(const float* f, bf8& hi, bf8& lo) {
  u32x4_t h, l;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const unsigned hw = pack_bf2(f[2 * i], f[2 * i + 1]);
    h[i] = hw;
    l[i] = pack_bf2(f[2 * i] - bf_lo(hw), f[2 * i + 1] - bf_hi(hw));
  }
  hi = __builtin_bit_cast(bf8, h);
  lo = __builtin_bit_cast(bf8, l);
}

}  // namespace
