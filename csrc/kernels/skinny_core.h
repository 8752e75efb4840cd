// Weight-streaming core of the bf16 decode GEMMs (skinny_gemm.hip, hybrid_skinny.hip): a workgroup of
// 8 waves computes 16 NC output channels for 16 MB token rows; wave w owns K part [w K / 8, (w + 1) K / 8)
// in 64-k chunks, two v_mfma_f32_16x16x32_bf16 each with the weights as the A operand.  Lane (c, g)
// reads 16 g .. 16 g + 15 of its chunk of weight row c and of token row c.
#pragma once

#include "common.h"

namespace mx {

typedef __bf16 bf16x8_sk __attribute__((ext_vector_type(8)));

__device__ __forceinline__ f32x4 mfma16_sk(const u16x8& a, const u16x8& b, const f32x4& c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_sk, a), __builtin_bit_cast(bf16x8_sk, b),
                                                 c, 0, 0, 0);
}

constexpr int kSkWaves = 8;
// 64-k chunks whose loads are issued before the first is used
constexpr int sk_unr(int nc) { return nc == 1 ? 8 : 4; }

// the first block of weight loads, issued ahead of a prologue that builds X in LDS
template <int NC>
__device__ __forceinline__ void sk_prefetch(const uint16_t* const (&wrow)[NC], int nit,
                                            u16x8 (&apre)[sk_unr(NC)][NC][2]) {
  constexpr int UNR = sk_unr(NC);
  if (nit >= UNR) {
#pragma unroll
    for (int u = 0; u < UNR; ++u)
#pragma unroll
      for (int j = 0; j < NC; ++j) {
        apre[u][j][0] = *reinterpret_cast<const u16x8*>(wrow[j] + u * 64);
        apre[u][j][1] = *reinterpret_cast<const u16x8*>(wrow[j] + u * 64 + 8);
      }
  }
}

// acc[j][mb] (zeroed here) = this wave's K part; PRE: apre holds the first block's weights
template <int MB, int NC, bool PRE>
__device__ __forceinline__ void sk_stream(const uint16_t* const (&wrow)[NC], const uint16_t* const (&xr)[MB], int nit,
                                          const u16x8 (&apre)[sk_unr(NC)][NC][2], f32x4 (&acc)[NC][MB]) {
  constexpr int UNR = sk_unr(NC);
#pragma unroll
  for (int j = 0; j < NC; ++j)
#pragma unroll
    for (int mb = 0; mb < MB; ++mb) acc[j][mb] = f32x4{0.f, 0.f, 0.f, 0.f};
  auto load = [&](int k, u16x8 (&a)[NC][2], u16x8 (&b)[MB][2]) {
#pragma unroll
    for (int j = 0; j < NC; ++j) {
      a[j][0] = *reinterpret_cast<const u16x8*>(wrow[j] + k);
      a[j][1] = *reinterpret_cast<const u16x8*>(wrow[j] + k + 8);
    }
#pragma unroll
    for (int mb = 0; mb < MB; ++mb) {
      b[mb][0] = *reinterpret_cast<const u16x8*>(xr[mb] + k);
      b[mb][1] = *reinterpret_cast<const u16x8*>(xr[mb] + k + 8);
    }
  };
  auto step = [&](const u16x8 (&a)[NC][2], const u16x8 (&b)[MB][2]) {
#pragma unroll
    for (int j = 0; j < NC; ++j)
#pragma unroll
      for (int mb = 0; mb < MB; ++mb) {
        acc[j][mb] = mfma16_sk(a[j][0], b[mb][0], acc[j][mb]);
        acc[j][mb] = mfma16_sk(a[j][1], b[mb][1], acc[j][mb]);
      }
  };
  int it = 0;
  if constexpr (PRE) {
    if (nit >= UNR) {  // first block: weights prefetched above, X fragments from LDS
      u16x8 b[UNR][MB][2];
#pragma unroll
      for (int u = 0; u < UNR; ++u)
#pragma unroll
        for (int mb = 0; mb < MB; ++mb) {
          b[u][mb][0] = *reinterpret_cast<const u16x8*>(xr[mb] + u * 64);
          b[u][mb][1] = *reinterpret_cast<const u16x8*>(xr[mb] + u * 64 + 8);
        }
#pragma unroll
      for (int u = 0; u < UNR; ++u) step(apre[u], b[u]);
      it = UNR;
    }
  }
  for (; it + UNR <= nit; it += UNR) {
    u16x8 a[UNR][NC][2], b[UNR][MB][2];
#pragma unroll
    for (int u = 0; u < UNR; ++u) load((it + u) * 64, a[u], b[u]);
#pragma unroll
    for (int u = 0; u < UNR; ++u) step(a[u], b[u]);
  }
  for (; it < nit; ++it) {
    u16x8 a[NC][2], b[MB][2];
    load(it * 64, a, b);
    step(a, b);
  }
}

}  // namespace mx
