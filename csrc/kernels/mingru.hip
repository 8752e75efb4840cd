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

// Tokens [t0, t0 + U) of NP projections (each W apart) of VEC channels, as stored; rows past n - 1
// repeat the last one (loaded, not used).
template <typename T, int VEC, int NP>
struct Batch {
  static constexpr int U = sizeof(T) == 2 ? 8 : 4;
  typedef T vt __attribute__((ext_vector_type(VEC > 1 ? VEC : 2)));
  vt r[U][NP];
  __device__ __forceinline__ void load(const T* p, int64_t ldx, int W, int t0, int n) {
#pragma unroll
    for (int j = 0; j < U; ++j) {
      const T* q = p + (int64_t)min(t0 + j, n - 1) * ldx;
#pragma unroll
      for (int k = 0; k < NP; ++k) {
        if constexpr (VEC > 1) r[j][k] = *reinterpret_cast<const vt*>(q + (int64_t)k * W);
        else r[j][k].x = q[(int64_t)k * W];
      }
    }
  }
  __device__ __forceinline__ void get(int j, int k, float (&v)[VEC]) const {
#pragma unroll
    for (int i = 0; i < VEC; ++i) {
      const T e = r[j][k][i];
      v[i] = ld1(&e);
    }
  }
};

// chunks [nc, 4] = (first row, rows, sequence, 1 for the sequence's last chunk)
template <typename T, int VEC>
__global__ void __launch_bounds__(64) mingru_reduce_kernel(const T* __restrict__ x, int64_t ldx,
                                                           const float* __restrict__ bias,
                                                           const int32_t* __restrict__ chunks, float* __restrict__ prod,
                                                           float* __restrict__ part, int W) {
  typedef Batch<T, VEC, 2> B;
  const int c = (blockIdx.x * 64 + threadIdx.x) * VEC, ck = blockIdx.y;
  if (c >= W || chunks[4 * ck + 3]) return;
  const int r0 = chunks[4 * ck], n = chunks[4 * ck + 1];
  float bz[VEC], bu[VEC], a[VEC], s[VEC];
  ldv<VEC>(bias + c, bz);
  ldv<VEC>(bias + W + c, bu);
#pragma unroll
  for (int i = 0; i < VEC; ++i) a[i] = 1.f, s[i] = 0.f;
  const T* p = x + (int64_t)r0 * ldx + c;
  auto work = [&](const B& q, int t0) {
#pragma unroll
    for (int j = 0; j < B::U; ++j) {
      if (t0 + j >= n) break;
      float z[VEC], u[VEC];
      q.get(j, 0, z);
      q.get(j, 1, u);
#pragma unroll
      for (int i = 0; i < VEC; ++i) {
        float keep, add;
        mingru_gate<T>(z[i] + bz[i], u[i] + bu[i], keep, add);
        a[i] *= keep;
        s[i] = keep * s[i] + add;
      }
    }
  };
  B q0, q1;  // one batch in flight while the other is folded in
  q0.load(p, ldx, W, 0, n);
  for (int t = 0; t < n; t += 2 * B::U) {
    if (t + B::U < n) q1.load(p, ldx, W, t + B::U, n);
    work(q0, t);
    if (t + 2 * B::U < n) q0.load(p, ldx, W, t + 2 * B::U, n);
    if (t + B::U < n) work(q1, t + B::U);
  }
  stv<VEC>(prod + (int64_t)ck * W + c, a);
  stv<VEC>(part + (int64_t)ck * W + c, s);
}

// seqs [n, 3] = (slot, first chunk, chunks): part[chunk] <- the state ahead of the chunk.  A workgroup
// takes 16 channels; its 16 thread groups compose 8 chunks each and meet in LDS, 128 chunks at a time.
__global__ void __launch_bounds__(256) mingru_carry_kernel(const int32_t* __restrict__ seqs,
                                                           const float* __restrict__ prod, float* __restrict__ part,
                                                           int W) {
  __shared__ float sa[16][16], sb[16][16];
  const int cl = threadIdx.x & 15, g = threadIdx.x >> 4, sq = blockIdx.y;
  const int c = blockIdx.x * 16 + cl;
  const bool on = c < W;
  const int c0 = seqs[3 * sq + 1], n = seqs[3 * sq + 2];
  float carry = 0.f;
  for (int k0 = 0; k0 < n; k0 += 128) {
    float a[8], b[8], A = 1.f, B = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int k = k0 + 8 * g + j;
      const bool live = on && k < n - 1;  // the last chunk is not reduced
      const int64_t o = (int64_t)(c0 + k) * W + c;
      a[j] = live ? prod[o] : 1.f;
      b[j] = live ? part[o] : 0.f;
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) A *= a[j], B = a[j] * B + b[j];
    sa[g][cl] = A;
    sb[g][cl] = B;
    __syncthreads();
    float s = carry;
    for (int k = 0; k < 16; ++k) {
      const float nx = sa[k][cl] * carry + sb[k][cl];
      carry = nx;
      if (k + 1 == g) s = nx;
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int k = k0 + 8 * g + j;
      if (on && k < n) part[(int64_t)(c0 + k) * W + c] = s;
      s = a[j] * s + b[j];
    }
    __syncthreads();
  }
}

template <typename T, int VEC>
__global__ void __launch_bounds__(64) mingru_replay_kernel(const T* __restrict__ x, int64_t ldx,
                                                           const float* __restrict__ bias,
                                                           const int32_t* __restrict__ chunks,
                                                           const int32_t* __restrict__ seqs,
                                                           const float* __restrict__ part, float* __restrict__ state,
                                                           T* __restrict__ y, int W) {
  typedef Batch<T, VEC, 3> B;
  const int c = (blockIdx.x * 64 + threadIdx.x) * VEC, ck = blockIdx.y;
  if (c >= W) return;
  const int r0 = chunks[4 * ck], n = chunks[4 * ck + 1], sq = chunks[4 * ck + 2];
  float bz[VEC], bu[VEC], s[VEC];
  const T* p = x + (int64_t)r0 * ldx + c;
  B q0, q1;
  q0.load(p, ldx, W, 0, n);
  ldv<VEC>(bias + c, bz);
  ldv<VEC>(bias + W + c, bu);
  if (ck == seqs[3 * sq + 1]) {
#pragma unroll
    for (int i = 0; i < VEC; ++i) s[i] = 0.f;
  } else {
    ldv<VEC>(part + (int64_t)ck * W + c, s);
  }
  T* o = y + (int64_t)r0 * W + c;
  auto work = [&](const B& q, int t0) {
#pragma unroll
    for (int j = 0; j < B::U; ++j) {
      if (t0 + j >= n) break;
      float z[VEC], u[VEC], g[VEC], out[VEC];
      q.get(j, 0, z);
      q.get(j, 1, u);
      q.get(j, 2, g);
#pragma unroll
      for (int i = 0; i < VEC; ++i) {
        float keep, add;
        mingru_gate<T>(z[i] + bz[i], u[i] + bu[i], keep, add);
        s[i] = keep * s[i] + add;
        out[i] = s[i] * (g[i] * sigmoid_t<T>(g[i]));
      }
      stv<VEC>(o + (int64_t)(t0 + j) * W, out);
    }
  };
  for (int t = 0; t < n; t += 2 * B::U) {
    if (t + B::U < n) q1.load(p, ldx, W, t + B::U, n);
    work(q0, t);
    if (t + 2 * B::U < n) q0.load(p, ldx, W, t + 2 * B::U, n);
    if (t + B::U < n) work(q1, t + B::U);
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
      mingru_carry_kernel<<<dim3((W + 15) / 16, nseq), 256, 0, stream>>>(seqs, prod, part, W);                   \
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
