// Torch op registrations of the serving kernels (decode attention, sampling, decode GEMMs).
#include "bindings_util.h"

namespace {

at::Tensor rope_append(const at::Tensor& qkv, const at::Tensor& cos, const at::Tensor& sin, const at::Tensor& pos,
                       const c10::optional<at::Tensor>& slots, at::Tensor k_cache, at::Tensor v_cache, int64_t Hq,
                       int64_t Hkv, int64_t D, const c10::optional<at::Tensor>& block_table) {
  check_bf16(qkv, "qkv");
  check_bf16(k_cache, "k_cache");
  check_bf16(v_cache, "v_cache");
  MX_CHECK(pos.scalar_type() == at::kInt, "pos int32");
  const int64_t B = qkv.size(0);
  MX_CHECK(qkv.size(1) == (Hq + 2 * Hkv) * D, "qkv width");
  MX_CHECK(k_cache.dim() == 4 && k_cache.size(1) == Hkv && k_cache.size(3) == D, "cache shape");
  DevGuard g(qkv.device());
  const int32_t* sl = nullptr;
  if (slots.has_value()) sl = slots->data_ptr<int32_t>();
  auto q = at::empty({B, Hq, D}, qkv.options());
  const KvPages pg = kv_pages(block_table, k_cache);
  MX_OK(mx_rope_append(bf(qkv), cos.data_ptr<float>(), sin.data_ptr<float>(), pos.data_ptr<int32_t>(), sl, bfm(q),
                       bfm(k_cache), bfm(v_cache), (int)B, (int)Hq, (int)Hkv, (int)D, (int)k_cache.size(2), pg.bt,
                       pg.maxb, cur_stream()));
  return q;
}

at::Tensor decode_attn(const at::Tensor& q, const at::Tensor& k_cache, const at::Tensor& v_cache,
                       const at::Tensor& lens, const c10::optional<at::Tensor>& slots, int64_t max_len, double scale,
                       int64_t len_off, const c10::optional<at::Tensor>& block_table,
                       const c10::optional<at::Tensor>& counters) {
  check_bf16(q, "q");
  MX_CHECK(lens.scalar_type() == at::kInt, "lens int32");
  const int64_t B = q.size(0), Hq = q.size(1), D = q.size(2);
  const int64_t Hkv = k_cache.size(1), max_seq = k_cache.size(2);
  DevGuard g(q.device());
  // counters: int32 [>= B * Hkv], zero, owned by the caller (a decode engine): the split
  // partials are merged in-launch by the last workgroup of each (seq, kv-head), which
  // resets its counter -> no combine launch (head_dim 128)
  unsigned int* cnt = nullptr;
  if (counters.has_value() && D == 128) {
    MX_CHECK(counters->scalar_type() == at::kInt && counters->is_contiguous() && counters->numel() >= B * Hkv &&
                 counters->device() == q.device(),
             "decode_attn: counters must be a contiguous int32 tensor of >= B * Hkv zeros on q's device");
    cnt = reinterpret_cast<unsigned int*>(counters->data_ptr<int32_t>());
  }
  const KvPages pg = kv_pages(block_table, k_cache);
  const int64_t cap = pg.bt ? (int64_t)pg.maxb * max_seq : max_seq;  // positions a sequence can hold
  const int64_t nsplit = std::max<int64_t>(1, (std::min(max_len, cap) + 255) / 256);
  auto ml = at::empty({B, Hq, nsplit, 2}, q.options().dtype(at::kFloat));
  auto po = at::empty({B, Hq, nsplit, D}, q.options().dtype(at::kFloat));
  auto out = at::empty({B, Hq * D}, q.options());
  const int32_t* sl = nullptr;
  if (slots.has_value()) sl = slots->data_ptr<int32_t>();
  MX_OK(mx_decode_attn(bf(q), bf(k_cache), bf(v_cache), lens.data_ptr<int32_t>(), (int)len_off, sl, ml.data_ptr<float>(),
                       po.data_ptr<float>(), bfm(out), (int)B, (int)Hq, (int)Hkv, (int)D, (int)max_seq, (int)nsplit,
                       (float)scale, pg.bt, pg.maxb, cnt, cur_stream()));
  return out;
}

// The split-K partials without the combine: (part_ml [B, Hq, nsplit, 2], part_o [B, Hq, nsplit, D]),
// merged by the o-projection's prologue (skinny_merge_linear, D = 128) or by attn_combine.
std::tuple<at::Tensor, at::Tensor> decode_attn_partials(const at::Tensor& q, const at::Tensor& k_cache,
                                                        const at::Tensor& v_cache, const at::Tensor& lens,
                                                        const c10::optional<at::Tensor>& slots, int64_t max_len,
                                                        double scale, int64_t len_off,
                                                        const c10::optional<at::Tensor>& block_table) {
  check_bf16(q, "q");
  MX_CHECK(lens.scalar_type() == at::kInt, "lens int32");
  const int64_t B = q.size(0), Hq = q.size(1), D = q.size(2);
  MX_CHECK(D == 128 || D == 64 || D == 32, "decode_attn_partials: head_dim 32, 64 or 128");
  const int64_t Hkv = k_cache.size(1), max_seq = k_cache.size(2);
  DevGuard g(q.device());
  const KvPages pg = kv_pages(block_table, k_cache);
  const int64_t cap = pg.bt ? (int64_t)pg.maxb * max_seq : max_seq;
  const int64_t nsplit = std::max<int64_t>(1, (std::min(max_len, cap) + 255) / 256);
  auto ml = at::empty({B, Hq, nsplit, 2}, q.options().dtype(at::kFloat));
  auto po = at::empty({B, Hq, nsplit, D}, q.options().dtype(at::kFloat));
  const int32_t* sl = nullptr;
  if (slots.has_value()) sl = slots->data_ptr<int32_t>();
  MX_OK(mx_decode_attn(bf(q), bf(k_cache), bf(v_cache), lens.data_ptr<int32_t>(), (int)len_off, sl, ml.data_ptr<float>(),
                       po.data_ptr<float>(), nullptr, (int)B, (int)Hq, (int)Hkv, (int)D, (int)max_seq, (int)nsplit,
                       (float)scale, pg.bt, pg.maxb, nullptr, cur_stream()));
  return {ml, po};
}

// y [M, N] = merge(part_ml, part_o) . W^T (decode o-projection with the split merge in the prologue)
at::Tensor skinny_merge_linear(const at::Tensor& ml, const at::Tensor& po, const at::Tensor& w) {
  MX_CHECK(ml.is_cuda() && ml.scalar_type() == at::kFloat && ml.is_contiguous() && ml.dim() == 4 && ml.size(3) == 2,
           "part_ml f32 [M, Hq, nsplit, 2]");
  MX_CHECK(po.is_cuda() && po.scalar_type() == at::kFloat && po.is_contiguous() && po.dim() == 4 &&
               po.size(0) == ml.size(0) && po.size(1) == ml.size(1) && po.size(2) == ml.size(2) && po.size(3) == 128,
           "part_o f32 [M, Hq, nsplit, 128]");
  MX_CHECK(w.is_cuda() && w.scalar_type() == at::kBFloat16 && w.dim() == 2 && w.stride(1) == 1, "w bf16 [N, K] rows");
  const int64_t M = ml.size(0), K = ml.size(1) * 128, N = w.size(0);
  MX_CHECK(w.size(1) == K, "w [N, Hq * 128]");
  DevGuard g(w.device());
  auto y = at::empty({M, N}, w.options());
  MX_OK(mx_skinny_merge_gemm(ml.data_ptr<float>(), po.data_ptr<float>(), (int)ml.size(2), bf(w), w.stride(0), bfm(y),
                             N, (int)M, (int)N, (int)K, cur_stream()));
  return y;
}

at::Tensor sample(const at::Tensor& logits, double temperature, int64_t seed, int64_t step) {
  MX_CHECK(logits.is_cuda() && logits.is_contiguous() && logits.dim() == 2, "logits [B, V] contiguous GPU");
  MX_CHECK(logits.scalar_type() == at::kBFloat16 || logits.scalar_type() == at::kFloat, "logits bf16/f32");
  DevGuard g(logits.device());
  auto out = at::empty({logits.size(0)}, logits.options().dtype(at::kLong));
  auto ws = at::empty({std::max<int64_t>(1, mx_sample_ws_floats((int)logits.size(0)))},
                      logits.options().dtype(at::kFloat));  // per-call partials (stream-ordered allocator)
  MX_OK(mx_sample(logits.data_ptr(), logits.scalar_type() == at::kBFloat16 ? 1 : 0, out.data_ptr<int64_t>(),
                  (int)logits.size(0), (int)logits.size(1), (float)temperature, (uint32_t)seed, (uint32_t)step,
                  ws.data_ptr<float>(), cur_stream()));
  return out;
}

// per-row temperature / seed / step without top-k / top-p (the split-vocabulary kernel of
// decode.hip; same draws as sample_rows for such rows)
at::Tensor sample_temp_rows(const at::Tensor& logits, const at::Tensor& temps, const at::Tensor& seeds,
                            const at::Tensor& steps) {
  MX_CHECK(logits.is_cuda() && logits.is_contiguous() && logits.dim() == 2, "logits [B, V] contiguous GPU");
  MX_CHECK(logits.scalar_type() == at::kBFloat16 || logits.scalar_type() == at::kFloat, "logits bf16/f32");
  const int64_t B = logits.size(0);
  auto chk = [&](const at::Tensor& t, at::ScalarType st, const char* name) {
    MX_CHECK(t.is_cuda() && t.is_contiguous() && t.scalar_type() == st && t.numel() == B, name);
  };
  chk(temps, at::kFloat, "temps f32 [B]");
  chk(seeds, at::kLong, "seeds i64 [B]");
  chk(steps, at::kInt, "steps i32 [B]");
  DevGuard g(logits.device());
  auto out = at::empty({B}, logits.options().dtype(at::kLong));
  auto ws = at::empty({std::max<int64_t>(1, mx_sample_ws_floats((int)B))}, logits.options().dtype(at::kFloat));
  MX_OK(mx_sample_temp_rows(logits.data_ptr(), logits.scalar_type() == at::kBFloat16 ? 1 : 0,
                            out.data_ptr<int64_t>(), (int)B, (int)logits.size(1), temps.data_ptr<float>(),
                            seeds.data_ptr<int64_t>(), steps.data_ptr<int32_t>(), ws.data_ptr<float>(),
                            cur_stream()));
  return out;
}

at::Tensor sample_rows(const at::Tensor& logits, const at::Tensor& temps, const at::Tensor& top_p,
                       const at::Tensor& top_k, const at::Tensor& seeds, const at::Tensor& steps) {
  MX_CHECK(logits.is_cuda() && logits.is_contiguous() && logits.dim() == 2, "logits [B, V] contiguous GPU");
  MX_CHECK(logits.scalar_type() == at::kBFloat16 || logits.scalar_type() == at::kFloat, "logits bf16/f32");
  const int64_t B = logits.size(0);
  auto chk = [&](const at::Tensor& t, at::ScalarType st, const char* name) {
    MX_CHECK(t.is_cuda() && t.is_contiguous() && t.scalar_type() == st && t.numel() == B, name);
  };
  chk(temps, at::kFloat, "temps f32 [B]");
  chk(top_p, at::kFloat, "top_p f32 [B]");
  chk(top_k, at::kInt, "top_k i32 [B]");
  chk(seeds, at::kLong, "seeds i64 [B]");
  chk(steps, at::kInt, "steps i32 [B]");
  DevGuard g(logits.device());
  auto out = at::empty({B}, logits.options().dtype(at::kLong));
  MX_OK(mx_sample_rows(logits.data_ptr(), logits.scalar_type() == at::kBFloat16 ? 1 : 0, out.data_ptr<int64_t>(),
                       (int)B, (int)logits.size(1), temps.data_ptr<float>(), top_p.data_ptr<float>(),
                       top_k.data_ptr<int32_t>(), seeds.data_ptr<int64_t>(), steps.data_ptr<int32_t>(),
                       cur_stream()));
  return out;
}



// ---------------------------------------------------------------- bf16 decode GEMM (serving)
// y[M, N] = x[M, K] . w[N, K]^T for M <= 32 tokens: the weight-streaming HIP kernel
// (csrc/kernels/skinny_gemm.hip).  Callers check the shape contract (mxllm/ops/linear.py).
at::Tensor skinny_linear(const at::Tensor& x, const at::Tensor& w) {
  MX_CHECK(x.is_cuda() && x.scalar_type() == at::kBFloat16 && x.dim() == 2 && x.stride(1) == 1, "x: bf16 [M, K] rows");
  MX_CHECK(w.is_cuda() && w.scalar_type() == at::kBFloat16 && w.dim() == 2 && w.stride(1) == 1, "w: bf16 [N, K] rows");
  const int64_t M = x.size(0), K = x.size(1), N = w.size(0);
  MX_CHECK(w.size(1) == K && M >= 1 && M <= 32 && N % 16 == 0 && K % 512 == 0 && x.stride(0) % 8 == 0 &&
               w.stride(0) % 8 == 0, "skinny_linear shape contract");
  DevGuard g(x.device());
  auto y = at::empty({M, N}, x.options());
  MX_OK(mx_skinny_gemm(bf(x), x.stride(0), bf(w), w.stride(0), bfm(y), N, (int)M, (int)N, (int)K, cur_stream()));
  return y;
}

// y[M, F] = swiglu(x[M, K] . w[2F, K]^T) for M <= 32 tokens, w = [gate; up] rows: the decode
// MLP's first projection with SwiGLU in the GEMM epilogue (csrc/kernels/skinny_gemm.hip).
at::Tensor skinny_linear_swiglu(const at::Tensor& x, const at::Tensor& w) {
  MX_CHECK(x.is_cuda() && x.scalar_type() == at::kBFloat16 && x.dim() == 2 && x.stride(1) == 1, "x: bf16 [M, K] rows");
  MX_CHECK(w.is_cuda() && w.scalar_type() == at::kBFloat16 && w.dim() == 2 && w.stride(1) == 1, "w: bf16 [2F, K] rows");
  const int64_t M = x.size(0), K = x.size(1), F = w.size(0) / 2;
  MX_CHECK(w.size(1) == K && w.size(0) == 2 * F && M >= 1 && M <= 32 && F % 8 == 0 && K % 512 == 0 &&
               x.stride(0) % 8 == 0 && w.stride(0) % 8 == 0, "skinny_linear_swiglu shape contract");
  DevGuard g(x.device());
  auto y = at::empty({M, F}, x.options());
  MX_OK(mx_skinny_gemm_swiglu(bf(x), x.stride(0), bf(w), w.stride(0), bfm(y), F, (int)M, (int)F, (int)K,
                              cur_stream()));
  return y;
}

// Decode rows (M <= 4): y = rmsnorm(h + delta) . w^T with the RMSNorm (and residual add) in the
// GEMM prologue (csrc/kernels/skinny_gemm.hip NORM); swiglu: w = [gate; up], y = silu(g) * u.
// Returns (y, h + delta) — the new residual is h itself when delta is absent.
std::tuple<at::Tensor, at::Tensor> skinny_norm_linear(const at::Tensor& h, const c10::optional<at::Tensor>& delta,
                                                      const at::Tensor& gamma, double eps, const at::Tensor& w,
                                                      bool swiglu) {
  MX_CHECK(h.is_cuda() && h.scalar_type() == at::kBFloat16 && h.dim() == 2 && h.stride(1) == 1, "h: bf16 [M, K] rows");
  MX_CHECK(w.is_cuda() && w.scalar_type() == at::kBFloat16 && w.dim() == 2 && w.stride(1) == 1, "w: bf16 [N, K] rows");
  const int64_t M = h.size(0), K = h.size(1), N = w.size(0);
  MX_CHECK(gamma.is_cuda() && gamma.scalar_type() == at::kBFloat16 && gamma.is_contiguous() && gamma.numel() == K,
           "gamma: bf16 [K]");
  MX_CHECK(w.size(1) == K && M >= 1 && M <= 4 && M * K <= 32768 && N % 16 == 0 && K % 512 == 0 &&
               h.stride(0) % 8 == 0 && w.stride(0) % 8 == 0 && (!swiglu || N % 16 == 0),
           "skinny_norm_linear shape contract");
  const uint16_t* dp = nullptr;
  int64_t ldd = 0;
  at::Tensor h_out = h;
  if (delta.has_value() && delta->defined()) {
    const at::Tensor& d = *delta;
    MX_CHECK(d.is_cuda() && d.scalar_type() == at::kBFloat16 && d.dim() == 2 && d.size(0) == M && d.size(1) == K &&
                 d.stride(1) == 1 && d.stride(0) % 8 == 0, "delta: bf16 [M, K] rows");
    dp = bf(d);
    ldd = d.stride(0);
    h_out = at::empty({M, K}, h.options());
  }
  DevGuard g(h.device());
  const int64_t Ny = swiglu ? N / 2 : N;
  auto y = at::empty({M, Ny}, h.options());
  MX_OK(mx_skinny_norm_gemm(bf(h), h.stride(0), dp, ldd, bf(gamma), (float)eps, dp ? bfm(h_out) : nullptr, bf(w),
                            w.stride(0), bfm(y), Ny, (int)M, (int)N, (int)K, swiglu ? 1 : 0, cur_stream()));
  return {y, h_out};
}

// Decode QKV projection with the RoPE / KV-cache append in the GEMM epilogue and, when gamma is
// given, the (residual-add +) RMSNorm in its prologue (csrc/kernels/skinny_gemm.hip ROPE / NORM).
// Returns (q [M, Hq, 128] rotated, new residual); K/V rows land in the caches at (slot, pos).
std::tuple<at::Tensor, at::Tensor> skinny_qkv_rope(const at::Tensor& h, const c10::optional<at::Tensor>& delta,
                                                   const c10::optional<at::Tensor>& gamma, double eps,
                                                   const at::Tensor& w, const at::Tensor& cosb, const at::Tensor& sinb,
                                                   const at::Tensor& pos, const c10::optional<at::Tensor>& slots,
                                                   at::Tensor& k_cache, at::Tensor& v_cache, int64_t Hq, int64_t Hkv,
                                                   const c10::optional<at::Tensor>& block_table) {
  MX_CHECK(h.is_cuda() && h.scalar_type() == at::kBFloat16 && h.dim() == 2 && h.stride(1) == 1, "h: bf16 [M, K] rows");
  MX_CHECK(w.is_cuda() && w.scalar_type() == at::kBFloat16 && w.dim() == 2 && w.stride(1) == 1, "w: bf16 [N, K] rows");
  const int64_t M = h.size(0), K = h.size(1);
  const bool norm = gamma.has_value() && gamma->defined();
  MX_CHECK(w.size(0) == (Hq + 2 * Hkv) * 128 && w.size(1) == K && M >= 1 && M <= (norm ? 4 : 16) && K % 512 == 0 &&
               (!norm || M * K <= 32768) && h.stride(0) % 8 == 0 && w.stride(0) % 8 == 0,
           "skinny_qkv_rope shape contract");
  MX_CHECK(cosb.scalar_type() == at::kFloat && sinb.scalar_type() == at::kFloat && cosb.is_contiguous() &&
               sinb.is_contiguous() && cosb.size(-1) == 64, "cos/sin f32 [max_pos, 64]");
  MX_CHECK(pos.scalar_type() == at::kInt && pos.numel() == M, "pos int32 [M]");
  check_bf16(k_cache, "k_cache");
  check_bf16(v_cache, "v_cache");
  MX_CHECK(k_cache.size(1) == Hkv && k_cache.size(3) == 128 && k_cache.is_contiguous() && v_cache.is_contiguous(),
           "caches [slots, Hkv, max_seq, 128]");
  const int32_t* sl = nullptr;
  if (slots.has_value() && slots->defined()) {
    MX_CHECK(slots->scalar_type() == at::kInt && slots->numel() == M, "slots int32 [M]");
    sl = slots->data_ptr<int32_t>();
  }
  const uint16_t* dp = nullptr;
  int64_t ldd = 0;
  at::Tensor h_out = h;
  if (norm && delta.has_value() && delta->defined()) {
    const at::Tensor& d = *delta;
    MX_CHECK(d.is_cuda() && d.scalar_type() == at::kBFloat16 && d.dim() == 2 && d.size(0) == M && d.size(1) == K &&
                 d.stride(1) == 1 && d.stride(0) % 8 == 0, "delta: bf16 [M, K] rows");
    dp = bf(d);
    ldd = d.stride(0);
    h_out = at::empty({M, K}, h.options());
  }
  if (norm)
    MX_CHECK(gamma->scalar_type() == at::kBFloat16 && gamma->is_contiguous() && gamma->numel() == K, "gamma bf16 [K]");
  DevGuard g(h.device());
  auto q = at::empty({M, Hq, 128}, h.options());
  const KvPages pg = kv_pages(block_table, k_cache);
  MX_OK(mx_skinny_rope_gemm(bf(h), h.stride(0), norm ? 1 : 0, dp, ldd, norm ? bf(*gamma) : nullptr, (float)eps,
                            dp ? bfm(h_out) : nullptr, bf(w), w.stride(0), cosb.data_ptr<float>(),
                            sinb.data_ptr<float>(), pos.data_ptr<int32_t>(), sl, bfm(q), bfm(k_cache),
                            bfm(v_cache), (int)Hq, (int)Hkv, (int)k_cache.size(2), pg.bt, pg.maxb, (int)M, (int)K, cur_stream()));
  return {q, h_out};
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(mxllm, m) {
  m.def("rope_append(Tensor qkv, Tensor cos, Tensor sin, Tensor pos, Tensor? slots, Tensor(a!) k_cache, Tensor(b!) v_cache, int Hq, int Hkv, int D, Tensor? block_table=None) -> Tensor");
  m.def("decode_attn(Tensor q, Tensor k_cache, Tensor v_cache, Tensor lens, Tensor? slots, int max_len, float scale, int len_off=0, Tensor? block_table=None, Tensor? counters=None) -> Tensor");
  m.def("decode_attn_partials(Tensor q, Tensor k_cache, Tensor v_cache, Tensor lens, Tensor? slots, int max_len, float scale, int len_off=0, Tensor? block_table=None) -> (Tensor, Tensor)");
  m.def("skinny_merge_linear(Tensor ml, Tensor po, Tensor w) -> Tensor");
  m.def("sample(Tensor logits, float temperature, int seed, int step) -> Tensor");
  m.def("sample_rows(Tensor logits, Tensor temps, Tensor top_p, Tensor top_k, Tensor seeds, Tensor steps) -> Tensor");
  m.def("sample_temp_rows(Tensor logits, Tensor temps, Tensor seeds, Tensor steps) -> Tensor");
  m.def("skinny_linear(Tensor x, Tensor w) -> Tensor");
  m.def("skinny_linear_swiglu(Tensor x, Tensor w) -> Tensor");
  m.def("skinny_qkv_rope(Tensor h, Tensor? delta, Tensor? gamma, float eps, Tensor w, Tensor cos, Tensor sin, Tensor pos, Tensor? slots, Tensor(a!) k_cache, Tensor(b!) v_cache, int Hq, int Hkv, Tensor? block_table=None) -> (Tensor, Tensor)");
  m.def("skinny_norm_linear(Tensor h, Tensor? delta, Tensor gamma, float eps, Tensor w, bool swiglu) -> (Tensor, Tensor)");
}

TORCH_LIBRARY_IMPL(mxllm, CUDA, m) {
  m.impl("rope_append", &rope_append);
  m.impl("decode_attn_partials", &decode_attn_partials);
  m.impl("skinny_merge_linear", &skinny_merge_linear);
  m.impl("decode_attn", &decode_attn);
  m.impl("sample", &sample);
  m.impl("sample_rows", &sample_rows);
  m.impl("sample_temp_rows", &sample_temp_rows);
  m.impl("skinny_linear", &skinny_linear);
  m.impl("skinny_linear_swiglu", &skinny_linear_swiglu);
  m.impl("skinny_qkv_rope", &skinny_qkv_rope);
  m.impl("skinny_norm_linear", &skinny_norm_linear);
}
