// minGRU recurrence for gfx950: S_t = (1 - z_t) S_(t-1) + z_t c_t per channel, f32 state, output
// S_t * silu(g_t).  Input rows hold the three projections z | u | g side by side; z and u get
// their bias here.
//
// Prompts: the recurrence is linear in S, so each sequence is cut into chunks.  One kernel reduces a
// chunk to (product of 1 - z, end state from zero), a second walks a sequence's chunks in order and
// leaves every chunk's start state, and a third replays the chunks from those and writes the
// outputs and the final state.  A sequence of one chunk needs the third only.  Threads own VEC
// neighbouring channels; a chunk's tokens are independent loads ahead of the serial f32 chain.
// Decode: one token per sequence, the state updated in place.
#include "hybrid.h"

namespace mx {

// chunks [nc, 4] = (first row, rows, sequence, 1 for the sequence's last chunk)
template <typename T, int VEC>
__global__ void __launch_bounds__(64) mingru_reduce_kernel(const T* __restrict__ x, int64_t ldx,
                                                           const float* __restrict__ bias,
                                                           const int32_t* __restrict__ chunks, float* __restrict__ prod,
                                                           float* __restrict__ part, int W) {
  const int c = (blockIdx.x * 64 + threadIdx.x) * VEC, ck = blockIdx.y;
  if (c >= W || chunks[4 * ck + 3]) return;
  const int r0 = chunks[4 * ck], n = chunks[4 * ck + 1];
  float bz[VEC], bu[VEC], a[VEC], s[VEC];
  ldv<VEC>(bias + c, bz);
  ldv<VEC>(bias + W + c, bu);
#pragma unroll
  for (int i = 0; i < VEC; ++i) a[i] = 1.f, s[i] = 0.f;
  const T* p = x + (int64_t)r0 * ldx + c;
#pragma unroll 4
  for (int t = 0; t < n; ++t) {
    float z[VEC], u[VEC];
    ldv<VEC>(p + (int64_t)t * ldx, z);
    ldv<VEC>(p + (int64_t)t * ldx + W, u);
#pragma unroll
    for (int i = 0; i < VEC; ++i) {
      float keep, add;
      mingru_gate<T>(z[i] + bz[i], u[i] + bu[i], keep, add);
      a[i] *= keep;
      s[i] = keep * s[i] + add;
    }
  }
  stv<VEC>(prod + (int64_t)ck * W + c, a);
  stv<VEC>(part + (int64_t)ck * W + c, s);
}

// seqs [n, 3] = (slot, first chunk, chunks): part[chunk] <- the state ahead of the chunk
__global__ void __launch_bounds__(64) mingru_carry_kernel(const int32_t* __restrict__ seqs,
                                                          const float* __restrict__ prod, float* __restrict__ part,
                                                          int W) {
  const int c = blockIdx.x * 64 + threadIdx.x, sq = blockIdx.y;
  if (c >= W) return;
  const int c0 = seqs[3 * sq + 1], n = seqs[3 * sq + 2];
  float s = 0.f;
  for (int k = 0; k < n; k += 8) {
    float a[8], b[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const bool on = k + j < n - 1;  // the last chunk's reduction is not formed
      const int64_t o = (int64_t)(c0 + (on ? k + j : 0)) * W + c;
      a[j] = on ? prod[o] : 0.f;
      b[j] = on ? part[o] : 0.f;
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      if (k + j < n) {
        part[(int64_t)(c0 + k + j) * W + c] = s;
        s = a[j] * s + b[j];
      }
    }
  }
}

template <typename T, int VEC>
__global__ void __launch_bounds__(64) mingru_replay_kernel(const T* __restrict__ x, int64_t ldx,
                                                           const float* __restrict__ bias,
                                                           const int32_t* __restrict__ chunks,
                                                           const int32_t* __restrict__ seqs,
                                                           const float* __restrict__ part, float* __restrict__ state,
                                                           T* __restrict__ y, int W) {
  const int c = (blockIdx.x * 64 + threadIdx.x) * VEC, ck = blockIdx.y;
  if (c >= W) return;
  const int r0 = chunks[4 * ck], n = chunks[4 * ck + 1], sq = chunks[4 * ck + 2];
  float bz[VEC], bu[VEC], s[VEC];
  ldv<VEC>(bias + c, bz);
  ldv<VEC>(bias + W + c, bu);
  if (ck == seqs[3 * sq + 1]) {
#pragma unroll
    for (int i = 0; i < VEC; ++i) s[i] = 0.f;
  } else {
    ldv<VEC>(part + (int64_t)ck * W + c, s);
  }
  const T* p = x + (int64_t)r0 * ldx + c;
  T* o = y + (int64_t)r0 * W + c;
#pragma unroll 4
  for (int t = 0; t < n; ++t) {
    float z[VEC], u[VEC], g[VEC], out[VEC];
    ldv<VEC>(p + (int64_t)t * ldx, z);
    ldv<VEC>(p + (int64_t)t * ldx + W, u);
    ldv<VEC>(p + (int64_t)t * ldx + 2 * W, g);
#pragma unroll
    for (int i = 0; i < VEC; ++i) {
      float keep, add;
      mingru_gate<T>(z[i] + bz[i], u[i] + bu[i], keep, add);
      s[i] = keep * s[i] + add;
      out[i] = s[i] * (g[i] * sigmoid_t<T>(g[i]));
    }
    stv<VEC>(o + (int64_t)t * W, out);
  }
  const int slot = seqs[3 * sq];
  if (chunks[4 * ck + 3] && slot >= 0) stv<VEC>(state + (int64_t)slot * W + c, s);
}

template <typename T, int VEC>
__global__ void __launch_bounds__(64) mingru_step_kernel(const T* __restrict__ x, int64_t ldx,
                                                         const float* __restrict__ bias,
                                                         const int32_t* __restrict__ slots, float* __restrict__ state,
                                                         T* __restrict__ y, int W) {
  const int c = (blockIdx.x * 64 + threadIdx.x) * VEC, b = blockIdx.y;
  if (c >= W) return;
  const T* p = x + (int64_t)b * ldx + c;
  float* sp = state + (int64_t)slots[b] * W + c;
  float bz[VEC], bu[VEC], s[VEC], z[VEC], u[VEC], g[VEC], out[VEC];
  ldv<VEC>(bias + c, bz);
  ldv<VEC>(bias + W + c, bu);
  ldv<VEC>(sp, s);
  ldv<VEC>(p, z);
  ldv<VEC>(p + W, u);
  ldv<VEC>(p + 2 * W, g);
#pragma unroll
  for (int i = 0; i < VEC; ++i) {
    float keep, add;
    mingru_gate<T>(z[i] + bz[i], u[i] + bu[i], keep, add);
    s[i] = keep * s[i] + add;
    out[i] = s[i] * (g[i] * sigmoid_t<T>(g[i]));
  }
  stv<VEC>(sp, s);
  stv<VEC>(y + (int64_t)b * W + c, out);
}

}  // namespace mx

using namespace mx;

// x [T, ldx] (z | u | g, each W wide), bias f32 [2 W] (z | u), y [T, W]; prod / part f32 [nc, W]
// scratch (may be null when every sequence is one chunk: multi = 0); state f32 [slots, W]
extern "C" int mx_mingru_scan(const void* x, int64_t ldx, int f32, const float* bias, const int32_t* chunks, int nc,
                              const int32_t* seqs, int nseq, int multi, float* prod, float* part, float* state,
                              void* y, int W, hipStream_t stream) {
  if (nc <= 0) return 0;
  if (W <= 0 || ldx < 3 * (int64_t)W || (multi && (!prod || !part)) || nc > 65535 || nseq > 65535) return -1;
  const bool v4 = W % 4 == 0 && ldx % 4 == 0;
#define MG(TT, VV)                                                                                              \
  {                                                                                                             \
    const dim3 grid((W + 64 * VV - 1) / (64 * VV), nc);                                                         \
    if (multi) {                                                                                                \
      mingru_reduce_kernel<TT, VV><<<grid, 64, 0, stream>>>((const TT*)x, ldx, bias, chunks, prod, part, W);    \
      mingru_carry_kernel<<<dim3((W + 63) / 64, nseq), 64, 0, stream>>>(seqs, prod, part, W);                   \
    }                                                                                                           \
    mingru_replay_kernel<TT, VV>                                                                                \
        <<<grid, 64, 0, stream>>>((const TT*)x, ldx, bias, chunks, seqs, part, state, (TT*)y, W);               \
  }
  if (f32) { if (v4) MG(float, 4) else MG(float, 1) }
  else { if (v4) MG(uint16_t, 4) else MG(uint16_t, 1) }
#undef MG
  return (int)hipGetLastError();
}

extern "C" int mx_mingru_step(const void* x, int64_t ldx, int f32, const float* bias, const int32_t* slots,
                              float* state, void* y, int B, int W, hipStream_t stream) {
  if (B <= 0) return 0;
  if (W <= 0 || ldx < 3 * (int64_t)W || B > 65535) return -1;
  const bool v4 = W % 4 == 0 && ldx % 4 == 0;
#define MS(TT, VV)                                                                                    \
  mingru_step_kernel<TT, VV><<<dim3((W + 64 * VV - 1) / (64 * VV), B), 64, 0, stream>>>(              \
      (const TT*)x, ldx, bias, slots, state, (TT*)y, W)
  if (f32) { if (v4) MS(float, 4); else MS(float, 1); }
  else { if (v4) MS(uint16_t, 4); else MS(uint16_t, 1); }
#undef MS
  return (int)hipGetLastError();
}
