// Row kernels of the recurrent / chunked-attention decoders for gfx950:
//   * embed_rows   : token rows of the embedding table into the f32 residual stream;
//   * group_norm   : (residual add +) RMS norm in equal consecutive groups, f32 residual;
//   * conv_rope    : short causal convolution over time on the q / k / v projections, rotation
//                    of interleaved pairs, and the KV-cache / convolution-tail stores (prompt
//                    rows of several sequences at once, or one token per sequence);
//   * poly_norm    : the polynomial-of-norms activation;
//   * attn_combine : split-K decode partials merged with the softmax sink and the output gate.
// Storage type T: bf16 (uint16_t) or float; every reduction, angle and product is f32.
#include <algorithm>

#include "conv_rope.h"
#include "hybrid.h"

namespace mx {

// ------------------------------------------------------------------ embedding -> f32 rows
template <typename T, int VEC>
__global__ void __launch_bounds__(256) embed_rows_kernel(const int64_t* __restrict__ ids, const T* __restrict__ w,
                                                         float* __restrict__ out, int64_t n, int W, int V) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= n) return;
  const int nv = W / VEC;
  const int64_t row = i / nv;
  const int c = (int)(i % nv) * VEC;
  int64_t id = ids[row];
  id = id < 0 ? 0 : (id >= V ? V - 1 : id);  // ids are checked on the host; stays in the table either way
  float v[VEC];
  ldv<VEC>(w + id * W + c, v);
  stv<VEC>(out + row * W + c, v);
}

// ------------------------------------------------------------------ grouped RMS norm
// The norm of a row in G equal parts is an RMS norm of G rows: one unit = one (row, part), held in
// registers by TPU threads (a wave or a workgroup).  h (f32, row stride W) += delta when given.
template <typename T, int TPU, int VEC>
__global__ void __launch_bounds__(TPU < 256 ? 256 : TPU)
    group_norm_kernel(const T* __restrict__ delta, int64_t ldd, float* __restrict__ h, const float* __restrict__ w,
                      T* __restrict__ y, int64_t ldy, int64_t units, int groups, int gs, float eps) {
  constexpr int ITERS = 16 / VEC;
  __shared__ float scratch[16];
  const int64_t unit = TPU < 256 ? (int64_t)blockIdx.x * (256 / TPU) + threadIdx.x / TPU : (int64_t)blockIdx.x;
  const bool on = unit < units;
  const int t = threadIdx.x % TPU;
  const int64_t row = on ? unit / groups : 0;
  const int g0 = on ? (int)(unit % groups) * gs : 0;
  float* hp = h + row * (int64_t)groups * gs + g0;
  const T* dp = delta ? delta + row * ldd + g0 : nullptr;
  float v[ITERS][VEC];
  float ss = 0.f;
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int c = (it * TPU + t) * VEC;
    if (on && c < gs) {
      ldv<VEC>(hp + c, v[it]);
      if (dp) {
        float d[VEC];
        ldv<VEC>(dp + c, d);
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[it][j] += d[j];
        stv<VEC>(hp + c, v[it]);
      }
#pragma unroll
      for (int j = 0; j < VEC; ++j) ss += v[it][j] * v[it][j];
    }
  }
  ss = TPU == 64 ? wave_sum(ss) : block_sum(ss, scratch);
  const float rs = 1.f / sqrtf(ss / (float)gs + eps);
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int c = (it * TPU + t) * VEC;
    if (on && c < gs) {
      float g[VEC], o[VEC];
      ldv<VEC>(w + g0 + c, g);
#pragma unroll
      for (int j = 0; j < VEC; ++j) o[j] = v[it][j] * rs * g[j];
      stv<VEC>(y + row * ldy + g0 + c, o);
    }
  }
}

// ------------------------------------------------------------------ convolution + rotation

// section and channel of flat vector index f: sec 0 q, 1 k, 2 v; head; d0; ch = flat channel
template <int VEC>
__device__ __forceinline__ void conv_where(const ConvRope& a, int f, int& sec, int& head, int& d0, int& ch, int& dim) {
  const int nd = (a.D + VEC - 1) / VEC, ne = (a.E + VEC - 1) / VEC;
  if (f < a.H * nd) {
    sec = 0, head = f / nd, d0 = (f % nd) * VEC, dim = a.D;
    ch = head * a.D + d0;
  } else if (f < (a.H + a.G) * nd) {
    f -= a.H * nd;
    sec = 1, head = f / nd, d0 = (f % nd) * VEC, dim = a.D;
    ch = a.H * a.D + head * a.D + d0;
  } else {
    f -= (a.H + a.G) * nd;
    sec = 2, head = f / ne, d0 = (f % ne) * VEC, dim = a.E;
    ch = (a.H + a.G) * a.D + head * a.E + d0;
  }
}

// values of channels [ch, ch + n) of a row; channels past n are 0 (n = VEC except at an odd head end)
template <int VEC, typename T>
__device__ __forceinline__ void ldn(const T* p, int n, float (&v)[VEC]) {
  if constexpr (VEC >= 4) {
    ldv<VEC>(p, v);
  } else {
#pragma unroll
    for (int i = 0; i < VEC; ++i) v[i] = i < n ? ld1(p + i) : 0.f;
  }
}
template <int VEC, typename T>
__device__ __forceinline__ void stn(T* p, int n, const float (&v)[VEC]) {
  if constexpr (VEC >= 4) {
    stv<VEC>(p, v);
  } else {
#pragma unroll
    for (int i = 0; i < VEC; ++i)
      if (i < n) st1(p + i, v[i]);
  }
}

// VEC channels of a row kept as stored (half the registers for bf16)
template <typename T, int VEC>
struct alignas(sizeof(T) * VEC) Piece {
  T e[VEC];
  __device__ __forceinline__ void load(const T* p, int n) {
    if constexpr (VEC >= 4) {
      typedef T vt __attribute__((ext_vector_type(VEC)));
      *reinterpret_cast<vt*>(e) = *reinterpret_cast<const vt*>(p);
    } else {
#pragma unroll
      for (int i = 0; i < VEC; ++i) e[i] = i < n ? p[i] : T(0);
    }
  }
  __device__ __forceinline__ void get(float (&v)[VEC]) const {
#pragma unroll
    for (int i = 0; i < VEC; ++i) v[i] = ld1(e + i);
  }
};

// rotate and store the convolved channels y of (row, position p); cr: the cache row (slot, head, p),
// or -1 (not kept)
template <int VEC, typename T>
__device__ __forceinline__ void conv_finish(const ConvRope& a, int sec, int head, int d0, int n, int64_t row, int p,
                                            int64_t cr, float (&y)[VEC]) {
  if (sec < 2 && d0 < a.rd) {
    const int64_t t = (int64_t)p * (a.rd >> 1) + (d0 >> 1);
    if constexpr (VEC == 8) {
      if ((a.rd & 7) == 0) {  // four whole pairs: 16-byte table reads
        float c[4], s[4];
        ldv<4>(a.cosb + t, c);
        ldv<4>(a.sinb + t, s);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float u = y[2 * i], v = y[2 * i + 1];
          y[2 * i] = u * c[i] - v * s[i];
          y[2 * i + 1] = v * c[i] + u * s[i];
        }
      }
    }
    if (VEC != 8 || (a.rd & 7)) {
#pragma unroll
      for (int i = 0; i + 1 < VEC; i += 2) {
        if (d0 + i + 1 < a.rd) {
          const float c = a.cosb[t + (i >> 1)], s = a.sinb[t + (i >> 1)];
          const float u = y[i], v = y[i + 1];
          y[i] = u * c - v * s;
          y[i + 1] = v * c + u * s;
        }
      }
    }
  }
  const int Wp = sec < 2 ? a.Dp : a.Ep;
  T* out = reinterpret_cast<T*>(sec == 0 ? a.q : sec == 1 ? a.k : a.v);
  if (out) {
    out += sec == 0 ? head * a.qh + row * a.qt : sec == 1 ? head * a.kh + row * a.kt : head * a.vh + row * a.vt;
    stn<VEC>(out + d0, n, y);
    const int dim = sec < 2 ? a.D : a.E;
    if (d0 + VEC >= dim)  // the head's last channels: its padding too
      for (int d = dim; d < Wp; ++d) st1(out + d, 0.f);
  }
  if (sec > 0 && cr >= 0) stn<VEC>(reinterpret_cast<T*>(sec == 1 ? a.kc : a.vc) + cr * Wp + d0, n, y);
}

// VEC consecutive channels of one tap's weights
template <int VEC>
__device__ __forceinline__ void conv_taps(const float* w, int n, float (&v)[VEC]) {
  ldn<VEC>(w, n, v);
}

// prompt rows: rows [T] = (position, slot or -1, sequence length, -).  One thread walks RUN consecutive
// rows of VEC channels with the last taps - 1 rows in registers.
constexpr int kConvRun = 4, kConvThreads = 128;
template <int VEC, typename T, int TAPS>
__global__ void __launch_bounds__(kConvThreads) conv_rope_prefill_kernel(ConvRope a, const int4* __restrict__ rows, int T_,
                                                                int nvec) {
  const int f = blockIdx.x * kConvThreads + threadIdx.x;
  if (f >= nvec) return;
  int sec, head, d0, ch, dim;
  conv_where<VEC>(a, f, sec, head, d0, ch, dim);
  const int n = min(VEC, dim - d0);
  const T* x = reinterpret_cast<const T*>(a.x) + ch;
  const int C = (a.H + a.G) * a.D + a.G * a.E;
  const int taps = TAPS ? TAPS : a.taps;
  const int r0 = blockIdx.y * kConvRun, r1 = min(T_, r0 + kConvRun);
  auto finish = [&](int r, const int4& ri, const float (&u)[VEC], float (&y)[VEC]) {
    const int p = ri.x, slot = ri.y, S = ri.z;
    int64_t cr = -1;
    if (slot >= 0 && a.kc) {
      if (p >= S - taps)
        stn<VEC>(reinterpret_cast<T*>(a.ring) + ((int64_t)slot * taps + p % taps) * C + ch, n, u);
      if (sec > 0 && p >= S / a.chunk * a.chunk)  // the chunk the next token belongs to
        cr = kv_row(a.bt, a.maxb, a.block, slot, a.G, head, p % a.chunk);
    }
    conv_finish<VEC, T>(a, sec, head, d0, n, r, p, cr, y);
  };
  if constexpr (TAPS > 0) {
    float wt[TAPS][VEC];
    Piece<T, VEC> win[TAPS - 1 + kConvRun];  // every row of the run and the ones ahead of it, in flight at once
#pragma unroll
    for (int j = 0; j < TAPS - 1 + kConvRun; ++j)
      win[j].load(x + min(max(r0 - (TAPS - 1) + j, 0), T_ - 1) * a.ldx, n);  // rows outside: not used
#pragma unroll
    for (int j = 0; j < TAPS; ++j) conv_taps<VEC>(a.w + (int64_t)j * C + ch, n, wt[j]);
    if constexpr (VEC == 8) {
      // the common run: whole rows inside one sequence, none of them among its last taps, all or none
      // kept, whole pairs of four: straight-line code, every table read independent of the row before
      const int4 ra = rows[r0], rb = rows[r1 - 1];
      const int p0 = ra.x, from = ra.z / a.chunk * a.chunk;
      const bool keep = ra.y >= 0 && a.kc && p0 >= from;
      if (r1 - r0 == kConvRun && p0 >= TAPS - 1 && rb.x == p0 + kConvRun - 1 && (a.rd & 7) == 0 && a.rd > 0 &&
          (ra.y < 0 || !a.kc || (rb.x < ra.z - taps && (keep || rb.x < from)))) {
        const bool rot = sec < 2 && d0 < a.rd;
        const int hr = a.rd >> 1, Wp = sec < 2 ? a.Dp : a.Ep;
        const float* ct = a.cosb + (int64_t)p0 * hr + (rot ? d0 >> 1 : 0);
        const float* st = a.sinb + (int64_t)p0 * hr + (rot ? d0 >> 1 : 0);
        const int64_t step = sec == 0 ? a.qt : sec == 1 ? a.kt : a.vt;
        T* out = reinterpret_cast<T*>(sec == 0 ? a.q : sec == 1 ? a.k : a.v) +
                 head * (sec == 0 ? a.qh : sec == 1 ? a.kh : a.vh) + r0 * step;
        const bool last = d0 + VEC >= dim && dim < Wp;
        auto run = [&](auto keep_c) {
#pragma unroll
          for (int k = 0; k < kConvRun; ++k) {
            float u[VEC], y[VEC], c[4], sn[4];
            ldv<4>(ct + (int64_t)k * hr, c);
            ldv<4>(st + (int64_t)k * hr, sn);
#pragma unroll
            for (int j = 0; j < TAPS; ++j) {
              win[k + j].get(u);
#pragma unroll
              for (int i = 0; i < VEC; ++i) y[i] = j == 0 ? wt[0][i] * u[i] : y[i] + wt[j][i] * u[i];
            }
#pragma unroll
            for (int i = 0; i < 4; ++i) {
              const float cc = rot ? c[i] : 1.f, ss = rot ? sn[i] : 0.f, e = y[2 * i], f = y[2 * i + 1];
              y[2 * i] = e * cc - f * ss;
              y[2 * i + 1] = f * cc + e * ss;
            }
            stv<VEC>(out + k * step + d0, y);
            if constexpr (decltype(keep_c)::value) {
              if (sec > 0)
                stv<VEC>(reinterpret_cast<T*>(sec == 1 ? a.kc : a.vc) +
                             kv_row(a.bt, a.maxb, a.block, ra.y, a.G, head, p0 - from + k) * Wp + d0,
                         y);
            }
          }
          if (last)  // the head's padding
            for (int k = 0; k < kConvRun; ++k)
              for (int d = dim; d < Wp; ++d) st1(out + k * step + d, 0.f);
        };
        if (keep) run(std::true_type{});
        else run(std::false_type{});
        return;
      }
    }
#pragma unroll
    for (int k = 0; k < kConvRun; ++k) {
      const int r = r0 + k;
      if (r >= r1) break;
      const int4 ri = rows[r];
      float u[VEC], y[VEC];
#pragma unroll
      for (int i = 0; i < VEC; ++i) y[i] = 0.f;
#pragma unroll
      for (int j = 0; j < TAPS; ++j) {
        if (ri.x < TAPS - 1 - j) continue;  // uniform: the row TAPS - 1 - j back is of an earlier sequence
        win[k + j].get(u);
#pragma unroll
        for (int i = 0; i < VEC; ++i) y[i] += wt[j][i] * u[i];
      }
      finish(r, ri, u, y);  // u: the row itself (the last tap)
    }
  } else {
    for (int r = r0; r < r1; ++r) {
      const int4 ri = rows[r];
      float y[VEC], u[VEC], wv[VEC];
#pragma unroll
      for (int i = 0; i < VEC; ++i) y[i] = 0.f;
      for (int j = 0; j < taps; ++j) {
        const int back = taps - 1 - j;
        if (ri.x < back) continue;
        ldn<VEC>(x + (int64_t)(r - back) * a.ldx, n, u);
        conv_taps<VEC>(a.w + (int64_t)j * C + ch, n, wv);
#pragma unroll
        for (int i = 0; i < VEC; ++i) y[i] += wv[i] * u[i];
      }
      finish(r, ri, u, y);  // u: the row itself (the last tap)
    }
  }
}

// one token per sequence: earlier projected values come from the ring
template <int VEC, typename T>
__global__ void __launch_bounds__(64) conv_rope_decode_kernel(ConvRope a, const int32_t* __restrict__ pos,
                                                              const int32_t* __restrict__ slots, int nvec) {
  const int f = blockIdx.x * 64 + threadIdx.x;
  if (f >= nvec) return;
  int sec, head, d0, ch, dim;
  conv_where<VEC>(a, f, sec, head, d0, ch, dim);
  const int n = min(VEC, dim - d0), b = blockIdx.y, p = pos[b], slot = slots[b];
  const int C = (a.H + a.G) * a.D + a.G * a.E;
  T* ring = reinterpret_cast<T*>(a.ring) + (int64_t)slot * a.taps * C + ch;
  float u[VEC], y[VEC];
  ldn<VEC>(reinterpret_cast<const T*>(a.x) + (int64_t)b * a.ldx + ch, n, u);
  float wv[VEC];
  conv_taps<VEC>(a.w + (int64_t)(a.taps - 1) * C + ch, n, wv);
#pragma unroll
  for (int i = 0; i < VEC; ++i) y[i] = wv[i] * u[i];
  for (int back = 1; back < a.taps && back <= p; ++back) {
    float o[VEC];
    ldn<VEC>(ring + (int64_t)((p - back) % a.taps) * C, n, o);
    conv_taps<VEC>(a.w + (int64_t)(a.taps - 1 - back) * C + ch, n, wv);
#pragma unroll
    for (int i = 0; i < VEC; ++i) y[i] += wv[i] * o[i];
  }
  stn<VEC>(ring + (int64_t)(p % a.taps) * C, n, u);
  conv_finish<VEC, T>(a, sec, head, d0, n, b, p,
                      sec > 0 ? kv_row(a.bt, a.maxb, a.block, slot, a.G, head, p % a.chunk) : -1, y);
}

// ------------------------------------------------------------------ PolyNorm
// y = a N(z) + b N(z^2) + c N(z^3) + e, N over the whole row; coef = (a, b, c, e).  One workgroup of
// NT threads per row; ITERS > 0: the row stays in registers (one read), 0: read twice.
template <typename T, int VEC, int NT, int ITERS>
__global__ void __launch_bounds__(NT) poly_norm_kernel(const T* __restrict__ z, int64_t ldz,
                                                       const float* __restrict__ coef, T* __restrict__ y, int F,
                                                       float eps) {
  __shared__ float red[3][16];
  constexpr int KEEP = ITERS > 0 ? ITERS : 1;
  typedef T vt __attribute__((ext_vector_type(VEC > 1 ? VEC : 2)));
  const T* zp = z + (int64_t)blockIdx.x * ldz;
  T* yp = y + (int64_t)blockIdx.x * F;
  float s1 = 0.f, s2 = 0.f, s3 = 0.f;
  auto add = [&](const float (&v)[VEC]) {
#pragma unroll
    for (int i = 0; i < VEC; ++i) {
      const float q = v[i] * v[i];
      s1 += q;
      s2 += q * q;
      s3 += q * q * q;
    }
  };
  vt keep[KEEP];
  if constexpr (ITERS > 0) {
#pragma unroll
    for (int it = 0; it < ITERS; ++it) {
      const int c = (it * NT + threadIdx.x) * VEC;
      if (c < F) keep[it] = *reinterpret_cast<const vt*>(zp + c);
      else keep[it] = 0;
    }
#pragma unroll
    for (int it = 0; it < ITERS; ++it) {
      float v[VEC];
      ldv<VEC>(reinterpret_cast<const T*>(&keep[it]), v);
      add(v);
    }
  } else {
    for (int c = threadIdx.x * VEC; c < F; c += NT * VEC) {
      float v[VEC];
      ldv<VEC>(zp + c, v);
      add(v);
    }
  }
  s1 = wave_sum(s1), s2 = wave_sum(s2), s3 = wave_sum(s3);
  if ((threadIdx.x & 63) == 0) red[0][threadIdx.x >> 6] = s1, red[1][threadIdx.x >> 6] = s2, red[2][threadIdx.x >> 6] = s3;
  __syncthreads();
  s1 = s2 = s3 = 0.f;
#pragma unroll
  for (int w = 0; w < NT / 64; ++w) s1 += red[0][w], s2 += red[1][w], s3 += red[2][w];
  const float inv = 1.f / (float)F;
  const float k1 = coef[0] / sqrtf(s1 * inv + eps), k2 = coef[1] / sqrtf(s2 * inv + eps),
              k3 = coef[2] / sqrtf(s3 * inv + eps), e = coef[3];
  auto put = [&](int c, const float (&v)[VEC]) {
    float o[VEC];
#pragma unroll
    for (int i = 0; i < VEC; ++i) o[i] = ((k3 * v[i] + k2) * v[i] + k1) * v[i] + e;
    stv<VEC>(yp + c, o);
  };
  if constexpr (ITERS > 0) {
#pragma unroll
    for (int it = 0; it < ITERS; ++it) {
      const int c = (it * NT + threadIdx.x) * VEC;
      float v[VEC];
      ldv<VEC>(reinterpret_cast<const T*>(&keep[it]), v);
      if (c < F) put(c, v);
    }
  } else {
    for (int c = threadIdx.x * VEC; c < F; c += NT * VEC) {
      float v[VEC];
      ldv<VEC>(zp + c, v);
      put(c, v);
    }
  }
}

// ------------------------------------------------------------------ decode combine: sink + gate
// out[b, h E + d] = sigmoid(gate[b, h E + d]) * sum_s 2^(m_s - M) o_s[d] / (2^-M + sum_s 2^(m_s - M) l_s)
// with M = max(0, m_s): the added 1 of the denominator is a key of score 0 without a value.
__global__ void __launch_bounds__(128) attn_combine_kernel(const float* __restrict__ ml, const float* __restrict__ po,
                                                           const uint16_t* __restrict__ gate, int64_t ldg,
                                                           uint16_t* __restrict__ out, int H, int D, int E,
                                                           int nsplit) {
  const int64_t bh = blockIdx.x, b = bh / H;
  const int h = (int)(bh % H), d = threadIdx.x;
  if (d >= E) return;
  const float* m = ml + bh * nsplit * 2;
  const float gv = bf2f(gate[b * ldg + (int64_t)h * E + d]);
  float M = 0.f;
  for (int s = 0; s < nsplit; ++s) M = fmaxf(M, m[2 * s]);
  float L = __builtin_amdgcn_exp2f(-M), acc = 0.f;
  for (int s = 0; s < nsplit; ++s) {
    const float ms = m[2 * s];
    if (ms == -INFINITY) continue;
    const float wg = __builtin_amdgcn_exp2f(ms - M);
    L += wg * m[2 * s + 1];
    acc += wg * po[(bh * nsplit + s) * D + d];
  }
  out[b * (int64_t)H * E + (int64_t)h * E + d] = f2bf(acc / L * sigmoid_t<uint16_t>(gv));
}

}  // namespace mx

using namespace mx;

extern "C" int mx_embed_rows(const int64_t* ids, const void* w, int f32, float* out, int64_t T, int W, int V,
                             hipStream_t stream) {
  if (T <= 0) return 0;
  if (W <= 0 || V <= 0) return -1;
  const int vec = W % 4 == 0 ? 4 : 1;
  const int64_t n = T * (W / vec);
  const unsigned grid = (unsigned)((n + 255) / 256);
#define EM(TT, VV) embed_rows_kernel<TT, VV><<<grid, 256, 0, stream>>>(ids, (const TT*)w, out, n, W, V)
  if (f32) { if (vec == 4) EM(float, 4); else EM(float, 1); }
  else { if (vec == 4) EM(uint16_t, 4); else EM(uint16_t, 1); }
#undef EM
  return (int)hipGetLastError();
}

extern "C" int mx_group_norm(const void* delta, int64_t ldd, float* h, const float* w, void* y, int64_t ldy, int f32,
                             int64_t T, int W, int groups, float eps, hipStream_t stream) {
  if (T <= 0) return 0;
  if (groups <= 0 || W % groups) return -1;
  const int gs = W / groups;
  if (gs > 16384) return -1;
  const int64_t units = T * groups;
  const bool v4 = gs % 4 == 0 && (!delta || ldd % 4 == 0) && ldy % 4 == 0;
#define GN(TT, TPU, VV)                                                                                      \
  group_norm_kernel<TT, TPU, VV>                                                                             \
      <<<(unsigned)(TPU == 64 ? (units + 3) / 4 : units), TPU == 64 ? 256 : TPU, 0, stream>>>(               \
          (const TT*)delta, ldd, h, w, (TT*)y, ldy, units, groups, gs, eps)
#define GNT(TT)                                                                                              \
  if (v4) { if (gs <= 512) GN(TT, 64, 4); else if (gs <= 4096) GN(TT, 256, 4); else GN(TT, 1024, 4); }       \
  else { if (gs <= 1024) GN(TT, 64, 1); else if (gs <= 4096) GN(TT, 256, 1); else GN(TT, 1024, 1); }
  if (f32) { GNT(float) } else { GNT(uint16_t) }
#undef GNT
#undef GN
  return (int)hipGetLastError();
}

static int conv_check(const ConvRope& a) {
  if (a.taps < 1 || a.H <= 0 || a.G <= 0 || a.H % a.G || a.D <= 0 || a.E <= 0 || a.rd < 0 || a.rd > a.D || a.rd % 2 ||
      a.chunk <= 0 || a.Dp < a.D || a.Ep < a.E || (a.kc && (!a.vc || !a.bt || a.block <= 0)))
    return -1;
  return 0;
}
template <int VEC>
static int conv_nvec(const ConvRope& a) {
  return (a.H + a.G) * ((a.D + VEC - 1) / VEC) + a.G * ((a.E + VEC - 1) / VEC);
}
static bool conv_v8(const ConvRope& a) {
  return a.D % 8 == 0 && a.E % 8 == 0 && a.ldx % 8 == 0 && a.Dp % 8 == 0 && a.Ep % 8 == 0 && a.qh % 8 == 0 &&
         a.qt % 8 == 0 && a.kh % 8 == 0 && a.kt % 8 == 0 && a.vh % 8 == 0 && a.vt % 8 == 0;
}


extern "C" int mx_conv_rope_prefill(const ConvRope* pa, int f32, const int32_t* rows, int T, hipStream_t stream) {
  if (T <= 0) return 0;
  const ConvRope& a = *pa;
  if (conv_check(a)) return -1;
#define CP(VV, TT, TP)                                                                             \
  conv_rope_prefill_kernel<VV, TT, TP><<<dim3((conv_nvec<VV>(a) + kConvThreads - 1) / kConvThreads, (T + kConvRun - 1) / kConvRun), kConvThreads, \
                                         0, stream>>>(a, (const int4*)rows, T, conv_nvec<VV>(a))
#define CPT(VV, TT)                                                                                \
  if (a.taps == 4) CP(VV, TT, 4); else if (a.taps == 3) CP(VV, TT, 3); else if (a.taps == 2) CP(VV, TT, 2); \
  else CP(VV, TT, 0)
  if (f32) { CPT(2, float); }
  else if (conv_v8(a)) { CPT(8, uint16_t); }
  else { CPT(2, uint16_t); }
#undef CPT
#undef CP
  return (int)hipGetLastError();
}

extern "C" int mx_conv_rope_decode(const ConvRope* pa, int f32, const int32_t* pos, const int32_t* slots, int B,
                                   hipStream_t stream) {
  if (B <= 0) return 0;
  const ConvRope& a = *pa;
  if (conv_check(a) || !a.ring) return -1;
#define CD(VV, TT)                                                                                          \
  conv_rope_decode_kernel<VV, TT><<<dim3((conv_nvec<VV>(a) + 63) / 64, B), 64, 0, stream>>>(a, pos, slots, \
                                                                                            conv_nvec<VV>(a))
  if (f32) CD(2, float);
  else if (conv_v8(a)) CD(8, uint16_t);
  else CD(2, uint16_t);
#undef CD
  return (int)hipGetLastError();
}

extern "C" int mx_poly_norm(const void* z, int64_t ldz, const float* coef, void* y, int f32, int64_t T, int F,
                            float eps, hipStream_t stream) {
  if (T <= 0) return 0;
  if (F <= 0) return -1;
  const unsigned g = (unsigned)T;
#define PN(TT, VV, NT, IT) poly_norm_kernel<TT, VV, NT, IT><<<g, NT, 0, stream>>>((const TT*)z, ldz, coef, (TT*)y, F, eps)
  if (f32) {
    if (F % 4 == 0 && ldz % 4 == 0) PN(float, 4, 256, 0); else PN(float, 1, 256, 0);
  } else if (F % 8 || ldz % 8) {
    PN(uint16_t, 1, 256, 0);
  } else if (T <= 64 && F > 4096) {  // decode rows: latency
    if (F <= 16384) PN(uint16_t, 8, 1024, 2); else if (F <= 32768) PN(uint16_t, 8, 1024, 4); else PN(uint16_t, 8, 1024, 0);
  } else if (F <= 4096) {
    PN(uint16_t, 8, 256, 2);
  } else if (F <= 16384) {
    PN(uint16_t, 8, 512, 4);
  } else if (F <= 32768) {
    PN(uint16_t, 8, 512, 8);
  } else {
    PN(uint16_t, 8, 256, 0);
  }
#undef PN
  return (int)hipGetLastError();
}

extern "C" int mx_attn_combine(const float* ml, const float* po, const uint16_t* gate, int64_t ldg, uint16_t* out,
                               int B, int H, int D, int E, int nsplit, hipStream_t stream) {
  if (B <= 0) return 0;
  if (E > 128 || E > D || nsplit < 1) return -1;
  attn_combine_kernel<<<B * H, 128, 0, stream>>>(ml, po, gate, ldg, out, H, D, E, nsplit);
  return (int)hipGetLastError();
}
