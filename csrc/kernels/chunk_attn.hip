// Attention inside chunks with a softmax sink and an output gate, any head sizes, bf16 or f32
// storage with f32 arithmetic (no matrix cores): the f32 serving path, and bf16 heads outside the
// MFMA kernels' sizes (attn_fwd.hip: up to 128 dims; decode.hip: up to 16 query heads per key head).
//
// One wave per (query row, head).  Keys go 64 at a time: lane l scores key l against the query in
// LDS, the tile's weights go to LDS, and lane l accumulates value dims l, l + 64, ...  The running
// maximum starts at 0 with a sum of 1: the added 1 of the denominator is a key of score 0 without a
// value.  Keys of row i are rows [i - (p mod chunk), i] of head-major prompt buffers, or cache rows
// [0, p mod chunk] of the sequence's slot.
#include "hybrid.h"

namespace mx {

constexpr int kCaMaxDim = 512;

template <typename T, bool CACHED>
__global__ void __launch_bounds__(64) chunk_attn_kernel(const T* __restrict__ q, int64_t qh, int64_t qt,
                                                        const T* __restrict__ k, const T* __restrict__ v, int64_t kh,
                                                        int64_t vh, int Dp, int Ep, const int32_t* __restrict__ pos,
                                                        const int32_t* __restrict__ slots,
                                                        const int32_t* __restrict__ bt, int maxb, int block,
                                                        const T* __restrict__ gate, int64_t ldg, T* __restrict__ out,
                                                        int H, int G, int D, int E, int chunk, float scale) {
  __shared__ float qs[kCaMaxDim];
  __shared__ float ps[64];
  const int row = blockIdx.x, h = blockIdx.y, g = h / (H / G), lane = threadIdx.x;
  const int n = pos[row] % chunk + 1;
  const T* qp = q + h * qh + row * qt;
  for (int d = lane; d < D; d += 64) qs[d] = ld1(qp + d) * scale;
  const int slot = CACHED ? slots[row] : 0;
  const T* kb = CACHED ? k : k + g * kh + (int64_t)(row - (n - 1)) * Dp;
  const T* vb = CACHED ? v : v + g * vh + (int64_t)(row - (n - 1)) * Ep;
  auto key_row = [&](int j) -> int64_t {
    if constexpr (CACHED) return kv_row(bt, maxb, block, slot, G, g, j);
    else return j;
  };
  float m = 0.f, l = 1.f, acc[kCaMaxDim / 64];
#pragma unroll
  for (int i = 0; i < kCaMaxDim / 64; ++i) acc[i] = 0.f;
  for (int j0 = 0; j0 < n; j0 += 64) {
    __syncthreads();  // the query is staged; the previous tile's weights are used up
    float s = -INFINITY;
    if (j0 + lane < n) {
      const T* kr = kb + key_row(j0 + lane) * Dp;
      s = 0.f;
      for (int d = 0; d < D; ++d) s += qs[d] * ld1(kr + d);
    }
    const float mn = fmaxf(m, wave_max(s));
    const float p = j0 + lane < n ? exp_t<T>(s - mn) : 0.f;
    const float al = exp_t<T>(m - mn);
    m = mn;
    l = l * al + wave_sum(p);
    ps[lane] = p;
    __syncthreads();
    const int nt = min(64, n - j0);
#pragma unroll
    for (int i = 0; i < kCaMaxDim / 64; ++i) acc[i] *= al;
    for (int j = 0; j < nt; ++j) {
      const T* vr = vb + key_row(j0 + j) * Ep;
      const float pj = ps[j];
#pragma unroll
      for (int i = 0; i < kCaMaxDim / 64; ++i)
        if (lane + 64 * i < E) acc[i] += pj * ld1(vr + lane + 64 * i);
    }
  }
  const float inv = 1.f / l;
#pragma unroll
  for (int i = 0; i < kCaMaxDim / 64; ++i) {
    const int e = lane + 64 * i;
    if (e < E)
      st1(out + (int64_t)row * H * E + (int64_t)h * E + e,
          acc[i] * inv * sigmoid_t<T>(ld1(gate + row * ldg + (int64_t)h * E + e)));
  }
}

}  // namespace mx

using namespace mx;

// prompt rows: q [H][rows] (strides qh, qt), k / v head-major (head strides kh / vh, row strides Dp /
// Ep); cached (slots given): k / v are the paged caches [blocks, G, block, Dp / Ep].  pos [rows].
extern "C" int mx_chunk_attn(const void* q, int64_t qh, int64_t qt, const void* k, const void* v, int64_t kh,
                             int64_t vh, int Dp, int Ep, const int32_t* pos, const int32_t* slots, const int32_t* bt,
                             int maxb, int block, const void* gate, int64_t ldg, void* out, int f32, int64_t rows,
                             int H, int G, int D, int E, int chunk, float scale, hipStream_t stream) {
  if (rows <= 0) return 0;
  if (H <= 0 || G <= 0 || H % G || D <= 0 || E <= 0 || D > kCaMaxDim || E > kCaMaxDim || chunk <= 0 || Dp < D ||
      Ep < E || H > 65535 || (slots && (!bt || block <= 0)))
    return -1;
  const dim3 grid((unsigned)rows, H);
#define CA(TT, CC)                                                                                                 \
  chunk_attn_kernel<TT, CC><<<grid, 64, 0, stream>>>((const TT*)q, qh, qt, (const TT*)k, (const TT*)v, kh, vh, Dp, \
                                                     Ep, pos, slots, bt, maxb, block, (const TT*)gate, ldg,        \
                                                     (TT*)out, H, G, D, E, chunk, scale)
  if (f32) { if (slots) CA(float, true); else CA(float, false); }
  else { if (slots) CA(uint16_t, true); else CA(uint16_t, false); }
#undef CA
  return (int)hipGetLastError();
}
