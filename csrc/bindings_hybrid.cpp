// Torch op registrations of the recurrent / chunked-attention decoder kernels (hybrid.hip, mingru.hip,
// chunk_attn.hip, attn_fwd.hip SEG).  Activations are bf16 or f32; norms, tables, biases, recurrent
// state and the residual stream are f32.
#include "bindings_util.h"
#include "kernels/conv_rope.h"

namespace {

bool act_f32(const at::Tensor& t, const char* name) {
  MX_CHECK(t.is_cuda(), name, " must be a GPU tensor");
  MX_CHECK(t.scalar_type() == at::kBFloat16 || t.scalar_type() == at::kFloat, name, " must be bf16 or f32");
  return t.scalar_type() == at::kFloat;
}
// a row-major (row-strided) 2-D activation; returns its row stride
int64_t act_rows(const at::Tensor& t, const char* name) {
  MX_CHECK(t.dim() == 2 && (t.stride(1) == 1 || t.size(1) == 1) && t.stride(0) >= t.size(1), name,
           " must be a row-major 2-D view");
  return t.stride(0);
}
const int32_t* i32(const at::Tensor& t, const char* name, int64_t n) {
  MX_CHECK(t.is_cuda() && t.scalar_type() == at::kInt && t.is_contiguous() && t.numel() >= n, name,
           " must be a contiguous int32 GPU tensor of at least ", n, " elements");
  return t.data_ptr<int32_t>();
}
// rows of 16-byte vector access: the data pointer (a view may start anywhere) decides as well as the stride
bool aligned16(const at::Tensor& t) { return (reinterpret_cast<uintptr_t>(t.data_ptr()) & 15) == 0; }

at::Tensor embed_rows(const at::Tensor& ids, const at::Tensor& w) {
  const bool f = act_f32(w, "w");
  MX_CHECK(ids.is_cuda() && ids.scalar_type() == at::kLong && ids.is_contiguous() && w.dim() == 2 && w.is_contiguous(),
           "embed_rows: ids int64, w [V, W] contiguous");
  DevGuard g(w.device());
  const int64_t T = ids.numel(), W = w.size(1);
  auto out = at::empty({T, W}, w.options().dtype(at::kFloat));
  MX_OK(mx_embed_rows(ids.data_ptr<int64_t>(), w.data_ptr(), f, out.data_ptr<float>(), T, (int)W, (int)w.size(0),
                      cur_stream()));
  return out;
}

// y = group_norm(h (+= delta)) * w in bf16 (or f32)
at::Tensor group_norm(const c10::optional<at::Tensor>& delta, at::Tensor h, const at::Tensor& w, int64_t groups,
                      double eps, bool f32) {
  check_f32(h, "h");
  check_f32(w, "w");
  MX_CHECK(h.dim() == 2 && w.numel() == h.size(1) && groups > 0 && h.size(1) % groups == 0, "group_norm shapes");
  DevGuard g(h.device());
  const int64_t T = h.size(0), W = h.size(1);
  auto y = at::empty({T, W}, h.options().dtype(f32 ? at::kFloat : at::kBFloat16));
  int64_t ldd = 0;
  const void* dp = nullptr;
  at::Tensor d;
  if (delta.has_value()) {
    d = *delta;
    MX_CHECK(act_f32(d, "delta") == f32, "delta has the output's type");
    ldd = act_rows(d, "delta");
    MX_CHECK(d.size(0) == T && d.size(1) == W, "delta shape");
    if (!aligned16(d)) d = d.clone(), ldd = W;
    dp = d.data_ptr();
  }
  MX_OK(mx_group_norm(dp, ldd, h.data_ptr<float>(), w.data_ptr<float>(), y.data_ptr(), W, f32, T, (int)W, (int)groups,
                      (float)eps, cur_stream()));
  return y;
}

// ---- fused decode GEMMs (hybrid_skinny.hip): bf16 rows, weights [N, K] with unit inner stride
struct HsIn {  // X = x, or group_norm(h + delta) * gamma with the new residual in h_out
  const uint16_t *x = nullptr, *delta = nullptr;
  const float *h = nullptr, *gamma = nullptr;
  float* h_out = nullptr;
  int64_t ldx = 0, ldd = 0, M = 0, K = 0;
  int norm = 0;
  at::Tensor hn;
};
HsIn hs_in(const at::Tensor& x, const c10::optional<at::Tensor>& delta, const c10::optional<at::Tensor>& gamma,
           const at::Tensor& w) {
  HsIn r;
  r.norm = gamma.has_value();
  r.M = x.size(0), r.K = x.size(1);
  MX_CHECK(w.is_cuda() && w.scalar_type() == at::kBFloat16 && w.dim() == 2 && w.stride(1) == 1 && w.size(1) == r.K &&
               aligned16(w) && aligned16(x) && x.dim() == 2, "fused decode GEMM: x [M, K], w bf16 [N, K]");
  if (!r.norm) {
    MX_CHECK(x.is_cuda() && x.scalar_type() == at::kBFloat16 && x.stride(1) == 1 && !delta.has_value(), "x bf16 rows");
    r.x = bf(x), r.ldx = x.stride(0);
    return r;
  }
  check_f32(x, "h");
  check_f32(*gamma, "gamma");
  MX_CHECK(gamma->numel() == r.K, "gamma [K]");
  r.h = x.data_ptr<float>(), r.gamma = gamma->data_ptr<float>();
  r.hn = x;
  if (delta.has_value()) {
    MX_CHECK(delta->is_cuda() && delta->scalar_type() == at::kBFloat16 && delta->sizes() == x.sizes() &&
                 delta->stride(1) == 1 && aligned16(*delta), "delta bf16 [M, K] rows");
    r.delta = bf(*delta), r.ldd = delta->stride(0);
    r.hn = at::empty_like(x);
    r.h_out = r.hn.data_ptr<float>();
  }
  return r;
}

// (group_norm(h + delta) * gamma) . w^T and the new residual
std::tuple<at::Tensor, at::Tensor> hs_norm_linear(const c10::optional<at::Tensor>& delta, const at::Tensor& h,
                                                  const at::Tensor& gamma, int64_t groups, double eps,
                                                  const at::Tensor& w) {
  DevGuard g(w.device());
  HsIn i = hs_in(h, delta, gamma, w);
  auto y = at::empty({i.M, w.size(0)}, w.options());
  MX_OK(mx_hs_norm_gemm(i.delta, i.ldd, i.h, i.gamma, i.h_out, (int)groups, (float)eps, bf(w), w.stride(0), bfm(y),
                        w.size(0), (int)i.M, (int)w.size(0), (int)i.K, cur_stream()));
  return {y, i.hn};
}

at::Tensor hs_poly_linear(const at::Tensor& z, const at::Tensor& coef, double eps, const at::Tensor& w) {
  DevGuard g(w.device());
  check_f32(coef, "coef");
  MX_CHECK(coef.numel() == 4, "four coefficients");
  HsIn i = hs_in(z, c10::nullopt, c10::nullopt, w);
  auto y = at::empty({i.M, w.size(0)}, w.options());
  MX_OK(mx_hs_poly_gemm(i.x, i.ldx, coef.data_ptr<float>(), (float)eps, bf(w), w.stride(0), bfm(y), w.size(0), (int)i.M,
                        (int)w.size(0), (int)i.K, cur_stream()));
  return y;
}

// x: bf16 rows, or with gamma the f32 residual; w [3 W, K]
std::tuple<at::Tensor, at::Tensor> hs_gru_linear(const c10::optional<at::Tensor>& delta, const at::Tensor& x,
                                                 const c10::optional<at::Tensor>& gamma, int64_t groups, double eps,
                                                 const at::Tensor& w, const at::Tensor& bias, const at::Tensor& slots,
                                                 at::Tensor state) {
  DevGuard g(w.device());
  HsIn i = hs_in(x, delta, gamma, w);
  const int64_t W = w.size(0) / 3;
  check_f32(bias, "bias");
  check_f32(state, "state");
  MX_CHECK(w.size(0) == 3 * W && bias.numel() == 2 * W && state.dim() == 2 && state.size(1) == W, "minGRU shapes");
  auto y = at::empty({i.M, W}, w.options());
  MX_OK(mx_hs_gru_gemm(i.x, i.ldx, i.norm, i.delta, i.ldd, i.h, i.gamma, i.h_out, (int)groups, (float)eps, bf(w),
                       w.stride(0), bias.data_ptr<float>(), i32(slots, "slots", i.M), state.data_ptr<float>(), bfm(y),
                       (int)i.M, (int)W, (int)i.K, cur_stream()));
  return {y, i.norm ? i.hn : x};
}

mx::ConvRope conv_args(const at::Tensor& x, const at::Tensor& w, const at::Tensor& cos, const at::Tensor& sin,
                       int64_t rd, int64_t H, int64_t G, int64_t D, int64_t E) {
  act_f32(x, "x");
  check_f32(w, "conv w");
  check_f32(cos, "cos");
  check_f32(sin, "sin");
  const int64_t C = (H + G) * D + G * E;
  MX_CHECK(w.dim() == 2 && w.size(1) == C, "conv w [taps, C]");
  MX_CHECK(cos.dim() == 2 && cos.size(1) == rd / 2 && sin.sizes() == cos.sizes(), "cos / sin [max_pos, rd / 2]");
  mx::ConvRope a = {};
  a.ldx = act_rows(x, "x");
  MX_CHECK(x.size(1) >= C && aligned16(x), "x [rows, >= C], 16-byte aligned");
  a.x = x.data_ptr();
  a.w = w.data_ptr<float>();
  a.taps = (int)w.size(0);
  a.cosb = cos.data_ptr<float>();
  a.sinb = sin.data_ptr<float>();
  a.rd = (int)rd, a.H = (int)H, a.G = (int)G, a.D = (int)D, a.E = (int)E;
  return a;
}

void conv_cache(mx::ConvRope& a, const at::Tensor& x, at::Tensor& kc, at::Tensor& vc, const at::Tensor& bt,
                at::Tensor& ring) {
  for (const at::Tensor& t : {kc, vc, ring})
    MX_CHECK(t.is_cuda() && t.is_contiguous() && t.scalar_type() == x.scalar_type(), "caches: contiguous, x's type");
  MX_CHECK(kc.dim() == 4 && vc.dim() == 4 && kc.size(1) == a.G && vc.size(1) == a.G && kc.size(2) == vc.size(2) &&
               kc.size(3) >= a.D && vc.size(3) >= a.E, "caches [blocks, G, block, >= dims]");
  MX_CHECK(ring.dim() == 3 && ring.size(1) == a.taps && ring.size(2) == (a.H + a.G) * a.D + a.G * a.E,
           "ring [slots, taps, C]");
  MX_CHECK(bt.is_cuda() && bt.scalar_type() == at::kInt && bt.dim() == 2 && bt.is_contiguous(), "block table");
  a.kc = kc.data_ptr(), a.vc = vc.data_ptr(), a.ring = ring.data_ptr();
  a.Dp = (int)kc.size(3), a.Ep = (int)vc.size(3);
  a.bt = bt.data_ptr<int32_t>(), a.maxb = (int)bt.size(1), a.block = (int)kc.size(2);
}

// -> q [H, T, Dp], k [G, T, Dp], v [G, T, Ep], convolved and rotated; padding dims are zero
std::tuple<at::Tensor, at::Tensor, at::Tensor> conv_rope_prefill(
    const at::Tensor& x, const at::Tensor& w, const at::Tensor& cos, const at::Tensor& sin, int64_t rd, int64_t H,
    int64_t G, int64_t D, int64_t E, int64_t Dp, int64_t Ep, const at::Tensor& rows, int64_t chunk, const c10::optional<at::Tensor>& kc, const c10::optional<at::Tensor>& vc,
    const c10::optional<at::Tensor>& bt, const c10::optional<at::Tensor>& ring) {
  DevGuard g(x.device());
  mx::ConvRope a = conv_args(x, w, cos, sin, rd, H, G, D, E);
  const int64_t T = x.size(0);
  MX_CHECK(Dp >= D && Ep >= E && chunk > 0 && chunk <= INT32_MAX && T <= INT32_MAX, "conv_rope sizes");
  auto q = at::empty({H, T, Dp}, x.options());
  auto k = at::empty({G, T, Dp}, x.options());
  auto v = at::empty({G, T, Ep}, x.options());
  a.q = q.data_ptr(), a.k = k.data_ptr(), a.v = v.data_ptr();
  a.qh = a.kh = T * Dp, a.qt = a.kt = Dp, a.vh = T * Ep, a.vt = Ep;
  a.Dp = (int)Dp, a.Ep = (int)Ep, a.chunk = (int)chunk;
  if (kc.has_value()) {
    MX_CHECK(vc.has_value() && bt.has_value() && ring.has_value(), "k / v caches, block table and ring together");
    at::Tensor kt = *kc, vt = *vc, rt = *ring;
    conv_cache(a, x, kt, vt, *bt, rt);
    MX_CHECK(a.Dp == Dp && a.Ep == Ep, "cache rows as wide as the outputs");
  }
  MX_OK(mx_conv_rope_prefill(&a, x.scalar_type() == at::kFloat, i32(rows, "rows", 4 * T), (int)T, cur_stream()));
  return {q, k, v};
}

// one token per sequence: q [B, H, Dp]; k / v appended to the caches, the projected values to the ring
at::Tensor conv_rope_decode(const at::Tensor& x, const at::Tensor& w, const at::Tensor& cos, const at::Tensor& sin,
                            int64_t rd, int64_t H, int64_t G, int64_t D, int64_t E, const at::Tensor& pos,
                            const at::Tensor& slots, int64_t chunk, at::Tensor kc, at::Tensor vc, const at::Tensor& bt,
                            at::Tensor ring) {
  DevGuard g(x.device());
  mx::ConvRope a = conv_args(x, w, cos, sin, rd, H, G, D, E);
  MX_CHECK(chunk > 0 && chunk <= INT32_MAX, "chunk");
  conv_cache(a, x, kc, vc, bt, ring);
  const int64_t B = x.size(0), Dp = a.Dp;
  auto q = at::empty({B, H, Dp}, x.options());
  a.q = q.data_ptr(), a.qh = Dp, a.qt = H * Dp, a.chunk = (int)chunk;
  MX_OK(mx_conv_rope_decode(&a, x.scalar_type() == at::kFloat, i32(pos, "pos", B), i32(slots, "slots", B), (int)B,
                            cur_stream()));
  return q;
}

// w [C + H E, K] (q | k | v | gate) -> (q [M, H, Dp], gate [M, H E], new residual)
std::tuple<at::Tensor, at::Tensor, at::Tensor> hs_conv_linear(
    const c10::optional<at::Tensor>& delta, const at::Tensor& x, const c10::optional<at::Tensor>& gamma,
    int64_t groups, double eps, const at::Tensor& w, const at::Tensor& cw, const at::Tensor& cos, const at::Tensor& sin,
    int64_t rd, int64_t H, int64_t G, int64_t D, int64_t E, const at::Tensor& pos, const at::Tensor& slots,
    int64_t chunk, at::Tensor kc, at::Tensor vc, const at::Tensor& bt, at::Tensor ring) {
  DevGuard g(w.device());
  HsIn i = hs_in(x, delta, gamma, w);
  mx::ConvRope a = {};
  check_f32(cw, "conv w");
  check_f32(cos, "cos");
  check_f32(sin, "sin");
  const int64_t C = (H + G) * D + G * E;
  MX_CHECK(cw.dim() == 2 && cw.size(1) == C && w.size(0) == C + H * E, "conv w [taps, C], w [C + H E, K]");
  MX_CHECK(cos.dim() == 2 && cos.size(1) == rd / 2 && sin.sizes() == cos.sizes(), "cos / sin [max_pos, rd / 2]");
  MX_CHECK(chunk > 0 && chunk <= INT32_MAX, "chunk");
  a.w = cw.data_ptr<float>(), a.taps = (int)cw.size(0);
  a.cosb = cos.data_ptr<float>(), a.sinb = sin.data_ptr<float>();
  a.rd = (int)rd, a.H = (int)H, a.G = (int)G, a.D = (int)D, a.E = (int)E, a.chunk = (int)chunk;
  conv_cache(a, w, kc, vc, bt, ring);
  auto q = at::empty({i.M, H, (int64_t)a.Dp}, w.options());
  auto gate = at::empty({i.M, H * E}, w.options());
  a.q = q.data_ptr(), a.qh = a.Dp, a.qt = H * a.Dp;
  MX_OK(mx_hs_conv_gemm(i.x, i.ldx, i.norm, i.delta, i.ldd, i.h, i.gamma, i.h_out, (int)groups, (float)eps, bf(w),
                        w.stride(0), &a, i32(pos, "pos", i.M), i32(slots, "slots", i.M), bfm(gate), (int)i.M, (int)i.K,
                        cur_stream()));
  return {q, gate, i.norm ? i.hn : x};
}

const void* gate_ptr(const at::Tensor& gate, const at::Tensor& like, int64_t rows, int64_t cols, int64_t& ld) {
  MX_CHECK(gate.is_cuda() && gate.scalar_type() == like.scalar_type(), "gate: q's type");
  ld = act_rows(gate, "gate");
  MX_CHECK(gate.size(0) == rows && gate.size(1) == cols, "gate [rows, H * E]");
  return gate.data_ptr();
}

// MFMA flash attention over a table of self-contained segments, with sink and gate (bf16)
at::Tensor attn_seg(const at::Tensor& q, const at::Tensor& k, const at::Tensor& v, const at::Tensor& blocks,
                    const at::Tensor& gate, int64_t E, double scale) {
  check_bf16(q, "q");
  check_bf16(k, "k");
  check_bf16(v, "v");
  MX_CHECK(q.dim() == 3 && k.dim() == 3 && v.sizes() == k.sizes() && k.size(1) == q.size(1) && k.size(2) == q.size(2),
           "q [H, T, D], k / v [G, T, D]");
  DevGuard g(q.device());
  const int64_t H = q.size(0), T = q.size(1), D = q.size(2), G = k.size(0);
  MX_CHECK(T * D * 2 < INT32_MAX, "attn_seg: too many rows for one pass");
  MX_CHECK(blocks.dim() == 2 && blocks.size(1) == 4, "blocks [n, 4]");
  const int32_t* bp = i32(blocks, "blocks", 4 * blocks.size(0));
  int64_t ldg = 0;
  const void* gp = gate_ptr(gate, q, T, H * E, ldg);
  auto o = at::empty({T, H * E}, q.options());
  MX_OK(mx_attn_fwd_seg(bf(q), bf(k), bf(v), bp, (int)blocks.size(0), (const uint16_t*)gp, ldg, bfm(o), (int)T, (int)H,
                        (int)G, (int)D, (int)E, (float)scale, cur_stream()));
  return o;
}

// attention of any head size without matrix cores.  Prompt rows: q [H, T, Dp], k [G, T, Dp], v [G, T, Ep];
// decode (slots and block table given): q [B, H, Dp] and the paged caches.
at::Tensor chunk_attn(const at::Tensor& q, const at::Tensor& k, const at::Tensor& v, const at::Tensor& pos,
                      const at::Tensor& gate, int64_t D, int64_t E, int64_t chunk, double scale,
                      const c10::optional<at::Tensor>& slots, const c10::optional<at::Tensor>& bt) {
  const bool f = act_f32(q, "q");
  const bool cached = slots.has_value();
  for (const at::Tensor& t : {q, k, v})
    MX_CHECK(t.is_contiguous() && t.scalar_type() == q.scalar_type() && t.dim() == (cached && !t.is_same(q) ? 4 : 3),
             "chunk_attn: contiguous q / k / v of one type");
  DevGuard g(q.device());
  const int64_t rows = q.size(cached ? 0 : 1), H = q.size(cached ? 1 : 0), Dp = q.size(2);
  const int64_t G = k.size(cached ? 1 : 0), Ep = v.size(-1);
  MX_CHECK(k.size(-1) == Dp && v.size(cached ? 1 : 0) == G && k.size(cached ? 2 : 1) == v.size(cached ? 2 : 1),
           "chunk_attn: k / v shapes");
  MX_CHECK(cached || k.size(1) == rows, "chunk_attn: one key per prompt row");
  MX_CHECK(chunk > 0 && chunk <= INT32_MAX, "chunk");
  const int32_t *sl = nullptr, *bp = nullptr;
  int maxb = 0, block = 0;
  if (cached) {
    MX_CHECK(bt.has_value() && bt->dim() == 2, "block table");
    sl = i32(*slots, "slots", rows);
    bp = i32(*bt, "block table", 1);
    maxb = (int)bt->size(1), block = (int)k.size(2);
  }
  int64_t ldg = 0;
  const void* gp = gate_ptr(gate, q, rows, H * E, ldg);
  auto o = at::empty({rows, H * E}, q.options());
  MX_OK(mx_chunk_attn(q.data_ptr(), cached ? Dp : rows * Dp, cached ? H * Dp : Dp, k.data_ptr(), v.data_ptr(),
                      rows * Dp, rows * Ep, (int)Dp, (int)Ep, i32(pos, "pos", rows), sl, bp, maxb, block, gp, ldg,
                      o.data_ptr(), f, rows, (int)H, (int)G, (int)D, (int)E, (int)chunk, (float)scale, cur_stream()));
  return o;
}

at::Tensor attn_combine(const at::Tensor& ml, const at::Tensor& po, const at::Tensor& gate, int64_t E) {
  check_f32(ml, "ml");
  check_f32(po, "po");
  MX_CHECK(ml.dim() == 4 && po.dim() == 4 && po.size(2) == ml.size(2) && po.size(1) == ml.size(1) &&
               po.size(0) == ml.size(0), "partials [B, H, splits, 2 / D]");
  DevGuard g(ml.device());
  const int64_t B = ml.size(0), H = ml.size(1);
  MX_CHECK(gate.is_cuda() && gate.scalar_type() == at::kBFloat16 && gate.size(0) == B && gate.size(1) == H * E,
           "gate bf16 [B, H * E]");
  const int64_t ldg = act_rows(gate, "gate");
  auto o = at::empty({B, H * E}, gate.options());
  MX_OK(mx_attn_combine(ml.data_ptr<float>(), po.data_ptr<float>(), bf(gate), ldg, bfm(o), (int)B, (int)H,
                        (int)po.size(3), (int)E, (int)ml.size(2), cur_stream()));
  return o;
}

// x [T, 3 W] (z | u | g) -> y [T, W]; state f32 [slots, W] gets each sequence's end state
at::Tensor mingru_scan(const at::Tensor& x, const at::Tensor& bias, const at::Tensor& chunks, const at::Tensor& seqs,
                       bool multi, const c10::optional<at::Tensor>& state) {
  const bool f = act_f32(x, "x");
  check_f32(bias, "bias");
  const int64_t ldx = act_rows(x, "x"), T = x.size(0), W = x.size(1) / 3;
  MX_CHECK(x.size(1) == 3 * W && bias.numel() == 2 * W && aligned16(x), "mingru: x [T, 3 W], bias [2 W]");
  MX_CHECK(chunks.dim() == 2 && chunks.size(1) == 4 && seqs.dim() == 2 && seqs.size(1) == 3, "mingru tables");
  DevGuard g(x.device());
  const int64_t nc = chunks.size(0), ns = seqs.size(0);
  float* sp = nullptr;
  at::Tensor st;
  if (state.has_value()) {
    st = *state;
    check_f32(st, "state");
    MX_CHECK(st.dim() == 2 && st.size(1) == W, "state [slots, W]");
    sp = st.data_ptr<float>();
  }
  at::Tensor prod, part;
  if (multi) {
    prod = at::empty({nc, W}, bias.options());
    part = at::empty({nc, W}, bias.options());
  }
  auto y = at::empty({T, W}, x.options());
  MX_OK(mx_mingru_scan(x.data_ptr(), ldx, f, bias.data_ptr<float>(), i32(chunks, "chunks", 4 * nc), (int)nc,
                       i32(seqs, "seqs", 3 * ns), (int)ns, multi, multi ? prod.data_ptr<float>() : nullptr,
                       multi ? part.data_ptr<float>() : nullptr, sp, y.data_ptr(), (int)W, cur_stream()));
  return y;
}

at::Tensor mingru_step(const at::Tensor& x, const at::Tensor& bias, const at::Tensor& slots, at::Tensor state) {
  const bool f = act_f32(x, "x");
  check_f32(bias, "bias");
  check_f32(state, "state");
  const int64_t ldx = act_rows(x, "x"), B = x.size(0), W = x.size(1) / 3;
  MX_CHECK(x.size(1) == 3 * W && bias.numel() == 2 * W && aligned16(x), "mingru: x [B, 3 W], bias [2 W]");
  MX_CHECK(state.dim() == 2 && state.size(1) == W, "state [slots, W]");
  DevGuard g(x.device());
  auto y = at::empty({B, W}, x.options());
  MX_OK(mx_mingru_step(x.data_ptr(), ldx, f, bias.data_ptr<float>(), i32(slots, "slots", B), state.data_ptr<float>(),
                       y.data_ptr(), (int)B, (int)W, cur_stream()));
  return y;
}

at::Tensor poly_norm(const at::Tensor& z, const at::Tensor& coef, double eps) {
  const bool f = act_f32(z, "z");
  check_f32(coef, "coef");
  MX_CHECK(coef.numel() == 4 && aligned16(z), "poly_norm: four coefficients");
  const int64_t ldz = act_rows(z, "z"), T = z.size(0), F = z.size(1);
  DevGuard g(z.device());
  auto y = at::empty({T, F}, z.options());
  MX_OK(mx_poly_norm(z.data_ptr(), ldz, coef.data_ptr<float>(), y.data_ptr(), f, T, (int)F, (float)eps, cur_stream()));
  return y;
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(mxllm, m) {
  m.def("embed_rows(Tensor ids, Tensor w) -> Tensor");
  m.def("group_norm(Tensor? delta, Tensor(a!) h, Tensor w, int groups, float eps, bool f32) -> Tensor");
  m.def("conv_rope_prefill(Tensor x, Tensor w, Tensor cos, Tensor sin, int rd, int H, int G, int D, int E, int Dp, int Ep, Tensor rows, int chunk, Tensor(a!)? kc=None, Tensor(b!)? vc=None, Tensor? bt=None, Tensor(c!)? ring=None) -> (Tensor, Tensor, Tensor)");
  m.def("conv_rope_decode(Tensor x, Tensor w, Tensor cos, Tensor sin, int rd, int H, int G, int D, int E, Tensor pos, Tensor slots, int chunk, Tensor(a!) kc, Tensor(b!) vc, Tensor bt, Tensor(c!) ring) -> Tensor");
  m.def("attn_seg(Tensor q, Tensor k, Tensor v, Tensor blocks, Tensor gate, int E, float scale) -> Tensor");
  m.def("chunk_attn(Tensor q, Tensor k, Tensor v, Tensor pos, Tensor gate, int D, int E, int chunk, float scale, Tensor? slots=None, Tensor? bt=None) -> Tensor");
  m.def("attn_combine(Tensor ml, Tensor po, Tensor gate, int E) -> Tensor");
  m.def("mingru_scan(Tensor x, Tensor bias, Tensor chunks, Tensor seqs, bool multi, Tensor(a!)? state=None) -> Tensor");
  m.def("mingru_step(Tensor x, Tensor bias, Tensor slots, Tensor(a!) state) -> Tensor");
  m.def("hs_norm_linear(Tensor? delta, Tensor h, Tensor gamma, int groups, float eps, Tensor w) -> (Tensor, Tensor)");
  m.def("hs_poly_linear(Tensor z, Tensor coef, float eps, Tensor w) -> Tensor");
  m.def("hs_gru_linear(Tensor? delta, Tensor x, Tensor? gamma, int groups, float eps, Tensor w, Tensor bias, Tensor slots, Tensor(a!) state) -> (Tensor, Tensor)");
  m.def("hs_conv_linear(Tensor? delta, Tensor x, Tensor? gamma, int groups, float eps, Tensor w, Tensor cw, Tensor cos, Tensor sin, int rd, int H, int G, int D, int E, Tensor pos, Tensor slots, int chunk, Tensor(a!) kc, Tensor(b!) vc, Tensor bt, Tensor(c!) ring) -> (Tensor, Tensor, Tensor)");
  m.def("poly_norm(Tensor z, Tensor coef, float eps) -> Tensor");
}

TORCH_LIBRARY_IMPL(mxllm, CUDA, m) {
  m.impl("embed_rows", &embed_rows);
  m.impl("group_norm", &group_norm);
  m.impl("conv_rope_prefill", &conv_rope_prefill);
  m.impl("conv_rope_decode", &conv_rope_decode);
  m.impl("attn_seg", &attn_seg);
  m.impl("chunk_attn", &chunk_attn);
  m.impl("attn_combine", &attn_combine);
  m.impl("mingru_scan", &mingru_scan);
  m.impl("mingru_step", &mingru_step);
  m.impl("hs_norm_linear", &hs_norm_linear);
  m.impl("hs_poly_linear", &hs_poly_linear);
  m.impl("hs_gru_linear", &hs_gru_linear);
  m.impl("hs_conv_linear", &hs_conv_linear);
  m.impl("poly_norm", &poly_norm);
}
