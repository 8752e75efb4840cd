// Fused decode GEMMs of the recurrent / chunked-attention decoders on the weight-streaming core
// (skinny_core.h), M <= 16 bf16 rows, Y = X . W^T:
//   prologues (the rows are rebuilt in LDS by every workgroup; M K <= 16384 for the norm, 32768 for PolyNorm):
//     kProNorm : X = group_norm(h + delta) * gamma, f32 residual; workgroup 0 stores h + delta;
//     kProPoly : X = poly_norm(z), the feed-forward activation ahead of the down projection;
//   epilogues:
//     kEpiPlain: Y bf16;
//     kEpiGru  : W = [z; u; g]: a workgroup's 16 weight rows are 4 channels of each (a quarter
//                idle), so the wave that sums the K parts holds z, u and g of its channels, advances
//                the f32 state and writes S * silu(g);
//     kEpiConv : W = [q; k; v; gate]: the causal convolution against the ring of earlier projected
//                values, the pair rotation and the KV-cache append on the 4 consecutive channels a
//                lane holds; the gate's channels go out as they are.
// Each replaces two to four launches of a decode step.
#include "conv_rope.h"
#include "hybrid.h"
#include "skinny_core.h"

namespace mx {

enum { kProNone, kProNorm, kProPoly };
enum { kEpiPlain, kEpiGru, kEpiConv };

struct HsNorm {
  const uint16_t* delta;  // [M, K] or nullptr
  int64_t ldd;
  const float* h;         // [M, K] f32 residual
  const float* gamma;     // [K]
  float* h_out;           // [M, K]: h + delta (when delta)
  int groups;
  float eps;
};
struct HsPoly {
  const float* coef;
  float eps;
};
struct HsGru {
  const float* bias;      // [2 W]: z | u
  const int32_t* slots;
  float* state;           // [slots, W]
  int W;
};
struct HsConv {
  ConvRope a;             // x unused; q [M, H, Dp]
  const int32_t* pos;
  const int32_t* slots;
  uint16_t* gate;         // [M, H E]
};

constexpr int kHsMaxChunks = 4;  // 8-element pieces per thread: M K <= 512 * 8 * 4

// rows of h (+ delta), normalised, into xs [M, K]: piece sums of squares, then one wave per (row, part)
__device__ __forceinline__ void hs_norm_rows(const HsNorm& na, int M, int K, uint16_t* xs, float* psum, float* rs) {
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  const int np = M * K / 8, gs = K / na.groups, per = gs / 8;
  float v[kHsMaxChunks][8];
#pragma unroll
  for (int i = 0; i < kHsMaxChunks; ++i) {
    const int p = i * 512 + tid;
    if (p < np) {
      const int m = p / (K / 8), c = (p % (K / 8)) * 8;
      ldv<8>(na.h + (int64_t)m * K + c, v[i]);
      if (na.delta) {
        float d[8];
        ldv<8>(na.delta + (int64_t)m * na.ldd + c, d);
#pragma unroll
        for (int j = 0; j < 8; ++j) v[i][j] += d[j];
        if (blockIdx.x == 0) stv<8>(na.h_out + (int64_t)m * K + c, v[i]);
      }
      float ss = 0.f;
#pragma unroll
      for (int j = 0; j < 8; ++j) ss += v[i][j] * v[i][j];
      psum[p] = ss;
    }
  }
  __syncthreads();
  for (int u = w; u < M * na.groups; u += kSkWaves) {  // part u: pieces [u per, (u + 1) per)
    float ss = 0.f;
    for (int i = lane; i < per; i += 64) ss += psum[u * per + i];
    ss = wave_sum(ss);
    if (lane == 0) rs[u] = 1.f / sqrtf(ss / (float)gs + na.eps);
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < kHsMaxChunks; ++i) {
    const int p = i * 512 + tid;
    if (p < np) {
      const int c = (p % (K / 8)) * 8;
      const float r = rs[p / per];
      float g[8], o[8];
      ldv<8>(na.gamma + c, g);
#pragma unroll
      for (int j = 0; j < 8; ++j) o[j] = v[i][j] * r * g[j];
      stv<8>(xs + (int64_t)p * 8, o);
    }
  }
  __syncthreads();
}

// poly_norm of the rows z [M, K] into xs [M, K]
__device__ __forceinline__ void hs_poly_rows(const uint16_t* __restrict__ z, int64_t ldz, const HsPoly& pp, int M, int K,
                                             uint16_t* xs, float (*red)[kSkWaves]) {
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  for (int m = 0; m < M; ++m) {
    float s[3] = {0.f, 0.f, 0.f};
    for (int c = tid * 8; c < K; c += 4096) {
      const u16x8 zv = *reinterpret_cast<const u16x8*>(z + (int64_t)m * ldz + c);
      *reinterpret_cast<u16x8*>(xs + (int64_t)m * K + c) = zv;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float v = bf2f(zv[j]), q = v * v;
        s[0] += q;
        s[1] += q * q;
        s[2] += q * q * q;
      }
    }
#pragma unroll
    for (int k = 0; k < 3; ++k) {
      s[k] = wave_sum(s[k]);
      if (lane == 0) red[k][w] = s[k];
    }
    __syncthreads();
    float kf[3];
#pragma unroll
    for (int k = 0; k < 3; ++k) {
      float t = 0.f;
#pragma unroll
      for (int i = 0; i < kSkWaves; ++i) t += red[k][i];
      kf[k] = pp.coef[k] / sqrtf(t / (float)K + pp.eps);
    }
    const float e = pp.coef[3];
    for (int c = tid * 8; c < K; c += 4096) {  // the pieces this thread stored
      u16x8* px = reinterpret_cast<u16x8*>(xs + (int64_t)m * K + c);
      const u16x8 zv = *px;
      u16x8 o;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float v = bf2f(zv[j]);
        o[j] = f2bf(((kf[2] * v + kf[1]) * v + kf[0]) * v + e);
      }
      *px = o;
    }
    __syncthreads();
  }
}

// lane (c, g): v[i] = projection g (z, u, gate) of channel 4 blk + i for token c
__device__ __forceinline__ void hs_gru_store(const f32x4& v, int lane, int M, int blk, const HsGru& gr, uint16_t* Y) {
  f32x4 u, gt;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    u[i] = __shfl(v[i], (lane & 15) + 16, 64);
    gt[i] = __shfl(v[i], (lane & 15) + 32, 64);
  }
  const int m = lane & 15, c = blk * 4;
  if (lane < 16 && m < M) {
    float* sp = gr.state + (int64_t)gr.slots[m] * gr.W + c;
    float bz[4], bu[4], s[4], o[4];
    ldv<4>(gr.bias + c, bz);
    ldv<4>(gr.bias + gr.W + c, bu);
    ldv<4>(sp, s);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      float keep, add;
      mingru_gate<uint16_t>(v[i] + bz[i], u[i] + bu[i], keep, add);
      s[i] = keep * s[i] + add;
      o[i] = s[i] * (gt[i] * sigmoid_t<uint16_t>(gt[i]));
    }
    stv<4>(sp, s);
    stv<4>(Y + (int64_t)m * gr.W + c, o);
  }
}

// v: channels [ch, ch + 4) of token m, all of one section and head
__device__ __forceinline__ void hs_conv_store(const f32x4& v, int ch, int m, int M, const HsConv& cv) {
  if (m >= M) return;
  const ConvRope& a = cv.a;
  const int qk = (a.H + a.G) * a.D, C = qk + a.G * a.E;
  float u[4], y[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) u[i] = bf2f(f2bf(v[i]));  // the projection as the ring stores it
  if (ch >= C) {
    stv<4>(cv.gate + (int64_t)m * a.H * a.E + (ch - C), u);
    return;
  }
  const int p = cv.pos[m], slot = cv.slots[m];
  uint16_t* ring = reinterpret_cast<uint16_t*>(a.ring) + (int64_t)slot * a.taps * C + ch;
  float wv[4];
  ldv<4>(a.w + (int64_t)(a.taps - 1) * C + ch, wv);
#pragma unroll
  for (int i = 0; i < 4; ++i) y[i] = wv[i] * u[i];
  for (int back = 1; back < a.taps && back <= p; ++back) {
    float o[4];
    ldv<4>(ring + (int64_t)((p - back) % a.taps) * C, o);
    ldv<4>(a.w + (int64_t)(a.taps - 1 - back) * C + ch, wv);
#pragma unroll
    for (int i = 0; i < 4; ++i) y[i] += wv[i] * o[i];
  }
  stv<4>(ring + (int64_t)(p % a.taps) * C, u);
  const int sec = ch < a.H * a.D ? 0 : ch < qk ? 1 : 2;
  const int rel = sec == 0 ? ch : sec == 1 ? ch - a.H * a.D : ch - qk;
  const int dim = sec < 2 ? a.D : a.E, Wp = sec < 2 ? a.Dp : a.Ep;
  const int head = rel / dim, d0 = rel % dim;
  if (sec < 2) {
#pragma unroll
    for (int i = 0; i < 4; i += 2) {
      if (d0 + i + 1 < a.rd) {
        const int64_t t = (int64_t)p * (a.rd >> 1) + ((d0 + i) >> 1);
        const float c = a.cosb[t], s = a.sinb[t], e = y[i], f = y[i + 1];
        y[i] = e * c - f * s;
        y[i + 1] = f * c + e * s;
      }
    }
  }
  if (sec == 0) {
    uint16_t* q = reinterpret_cast<uint16_t*>(a.q) + head * a.qh + (int64_t)m * a.qt;
    stv<4>(q + d0, y);
    if (d0 + 4 >= dim)
      for (int d = dim; d < Wp; ++d) q[d] = 0;
  } else {
    uint16_t* cache = reinterpret_cast<uint16_t*>(sec == 1 ? a.kc : a.vc);
    stv<4>(cache + kv_row(a.bt, a.maxb, a.block, slot, a.G, head, p % a.chunk) * Wp + d0, y);
  }
}

template <int PRO, int EPI>
__global__ void __launch_bounds__(512) hybrid_skinny_kernel(const uint16_t* __restrict__ X, int64_t ldx,
                                                            const uint16_t* __restrict__ W, int64_t ldw,
                                                            uint16_t* __restrict__ Y, int64_t ldy, int M, int K,
                                                            HsNorm na, HsPoly pp, HsGru gr, HsConv cv) {
  __shared__ f32x4 red[kSkWaves][64];
  const int tid = threadIdx.x, lane = tid & 63;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int c = lane & 15, g = lane >> 4;
  const int blk = blockIdx.x, kq = K / kSkWaves, nit = kq / 64;
  const int64_t row = EPI == kEpiGru ? (int64_t)min(c >> 2, 2) * gr.W + blk * 4 + (c & 3) : (int64_t)blk * 16 + c;
  const uint16_t* wrow[1] = {W + row * ldw + (int64_t)w * kq + 16 * g};
  const uint16_t* xr[1];
  u16x8 apre[sk_unr(1)][1][2];
  if constexpr (PRO != kProNone) {
    extern __shared__ __attribute__((aligned(16))) uint16_t xs[];  // [M, K], then the norm's scratch
    sk_prefetch<1>(wrow, nit, apre);
    if constexpr (PRO == kProNorm) {
      float* psum = reinterpret_cast<float*>(xs + (int64_t)M * K);
      hs_norm_rows(na, M, K, xs, psum, psum + M * K / 8);
    } else {
      __shared__ float pred[3][kSkWaves];
      hs_poly_rows(X, ldx, pp, M, K, xs, pred);
    }
    xr[0] = xs + (int64_t)min(c, M - 1) * K + (int64_t)w * kq + 16 * g;
  } else {
    xr[0] = X + (int64_t)min(c, M - 1) * ldx + (int64_t)w * kq + 16 * g;
  }
  f32x4 acc[1][1];
  sk_stream<1, 1, PRO != kProNone>(wrow, xr, nit, apre, acc);
  red[w][lane] = acc[0][0];
  __syncthreads();
  if (w == 0) {
    f32x4 s = red[0][lane];
#pragma unroll
    for (int ww = 1; ww < kSkWaves; ++ww) s += red[ww][lane];
    if constexpr (EPI == kEpiGru) {
      hs_gru_store(s, lane, M, blk, gr, Y);
    } else if constexpr (EPI == kEpiConv) {
      hs_conv_store(s, blk * 16 + 4 * g, c, M, cv);
    } else if (c < M) {
      u16x4 o;
#pragma unroll
      for (int i = 0; i < 4; ++i) o[i] = f2bf(s[i]);
      *reinterpret_cast<u16x4*>(Y + (int64_t)c * ldy + blk * 16 + 4 * g) = o;
    }
  }
}

static int hs_check(const uint16_t* x, int64_t ldx, int64_t ldw, int M, int K, int N) {
  if (M > 16 || K % 512 || ldw % 8 || ldw < K || N <= 0) return -1;
  if (x && (ldx % 8 || ldx < K)) return -1;
  return 0;
}
static int hs_norm_check(const HsNorm& na, int M, int K) {
  if (na.groups <= 0 || K % na.groups || (K / na.groups) % 8 || (int64_t)M * K > 512 * 8 * kHsMaxChunks ||
      M * na.groups > 512 || (na.delta && (na.ldd % 8 || na.ldd < K || !na.h_out)))
    return -1;
  return 0;
}
static size_t hs_norm_lds(int M, int K, int groups) { return (size_t)M * K * 2 + (size_t)M * K / 2 + (size_t)M * groups * 4; }

}  // namespace mx

using namespace mx;

// Common to the three: norm != 0: X = group_norm(h + delta) * gamma (x unused), else X = x bf16 rows.

// y [M, N] bf16
extern "C" int mx_hs_norm_gemm(const uint16_t* delta, int64_t ldd, const float* h, const float* gamma, float* h_out,
                               int groups, float eps, const uint16_t* w, int64_t ldw, uint16_t* y, int64_t ldy, int M,
                               int N, int K, hipStream_t stream) {
  if (M <= 0) return 0;
  const HsNorm na{delta, ldd, h, gamma, h_out, groups, eps};
  if (hs_check(nullptr, 0, ldw, M, K, N) || hs_norm_check(na, M, K) || N % 16 || ldy % 4 || ldy < N) return -1;
  hybrid_skinny_kernel<kProNorm, kEpiPlain><<<N / 16, 512, hs_norm_lds(M, K, groups), stream>>>(
      nullptr, 0, w, ldw, y, ldy, M, K, na, {}, {}, {});
  return (int)hipGetLastError();
}

// y [M, N] = poly_norm(z) . w^T
extern "C" int mx_hs_poly_gemm(const uint16_t* z, int64_t ldz, const float* coef, float eps, const uint16_t* w,
                               int64_t ldw, uint16_t* y, int64_t ldy, int M, int N, int K, hipStream_t stream) {
  if (M <= 0) return 0;
  if (hs_check(z, ldz, ldw, M, K, N) || (int64_t)M * K > 32768 || N % 16 || ldy % 4 || ldy < N) return -1;
  hybrid_skinny_kernel<kProPoly, kEpiPlain><<<N / 16, 512, (size_t)M * K * 2, stream>>>(
      z, ldz, w, ldw, y, ldy, M, K, {}, HsPoly{coef, eps}, {}, {});
  return (int)hipGetLastError();
}

// w [3 W, K] -> y [M, W] = S * silu(g), state advanced
extern "C" int mx_hs_gru_gemm(const uint16_t* x, int64_t ldx, int norm, const uint16_t* delta, int64_t ldd,
                              const float* h, const float* gamma, float* h_out, int groups, float eps,
                              const uint16_t* w, int64_t ldw, const float* bias, const int32_t* slots, float* state,
                              uint16_t* y, int M, int W, int K, hipStream_t stream) {
  if (M <= 0) return 0;
  const HsNorm na{delta, ldd, h, gamma, h_out, groups, eps};
  if (hs_check(norm ? nullptr : x, ldx, ldw, M, K, W) || W % 4 || (norm && hs_norm_check(na, M, K)) || (!norm && !x))
    return -1;
  const HsGru gr{bias, slots, state, W};
  if (norm)
    hybrid_skinny_kernel<kProNorm, kEpiGru><<<W / 4, 512, hs_norm_lds(M, K, groups), stream>>>(
        nullptr, 0, w, ldw, y, W, M, K, na, {}, gr, {});
  else
    hybrid_skinny_kernel<kProNone, kEpiGru><<<W / 4, 512, 0, stream>>>(x, ldx, w, ldw, y, W, M, K, {}, {}, gr, {});
  return (int)hipGetLastError();
}

// w [C + H E, K] -> q [M, H, Dp] (in a), k / v cache rows, ring, gate [M, H E]
extern "C" int mx_hs_conv_gemm(const uint16_t* x, int64_t ldx, int norm, const uint16_t* delta, int64_t ldd,
                               const float* h, const float* gamma, float* h_out, int groups, float eps,
                               const uint16_t* w, int64_t ldw, const ConvRope* pa, const int32_t* pos,
                               const int32_t* slots, uint16_t* gate, int M, int K, hipStream_t stream) {
  if (M <= 0) return 0;
  const HsNorm na{delta, ldd, h, gamma, h_out, groups, eps};
  const ConvRope& a = *pa;
  const int N = (a.H + a.G) * a.D + a.G * a.E + a.H * a.E;
  if (hs_check(norm ? nullptr : x, ldx, ldw, M, K, N) || (norm && hs_norm_check(na, M, K)) || (!norm && !x)) return -1;
  if (N % 16 || a.D % 4 || a.E % 4 || a.Dp % 4 || a.Ep % 4 || a.rd % 2 || a.rd > a.D || a.H <= 0 || a.G <= 0 ||
      a.H % a.G || a.taps < 1 || a.chunk <= 0 || a.block <= 0 || !a.ring || !a.kc || !a.vc || !a.bt || a.Dp < a.D ||
      a.Ep < a.E)
    return -1;
  const HsConv cv{a, pos, slots, gate};
  if (norm)
    hybrid_skinny_kernel<kProNorm, kEpiConv><<<N / 16, 512, hs_norm_lds(M, K, groups), stream>>>(
        nullptr, 0, w, ldw, nullptr, 0, M, K, na, {}, {}, cv);
  else
    hybrid_skinny_kernel<kProNone, kEpiConv><<<N / 16, 512, 0, stream>>>(x, ldx, w, ldw, nullptr, 0, M, K, {}, {}, {},
                                                                           cv);
  return (int)hipGetLastError();
}
