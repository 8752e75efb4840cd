// Helpers of the torch op registration files (bindings*.cpp): argument checks, the current HIP stream.
#pragma once

#include <torch/library.h>
#include <ATen/ATen.h>
#include <ATen/hip/impl/HIPStreamMasqueradingAsCUDA.h>
#include <ATen/hip/impl/HIPGuardImplMasqueradingAsCUDA.h>
#include <hip/hip_runtime.h>
#include "bindings.h"
#include <algorithm>
#include <vector>

namespace {

// On ROCm builds torch devices are DeviceType::CUDA backed by HIP: use the
// "masquerading" guard/stream so device indices and the current stream match torch's.
inline hipStream_t cur_stream() { return c10::hip::getCurrentHIPStreamMasqueradingAsCUDA().stream(); }
using DevGuard = c10::hip::HIPGuardMasqueradingAsCUDA;

#define MX_CHECK(cond, ...) TORCH_CHECK(cond, "mxllm: ", __VA_ARGS__)
#define MX_OK(call)                                                                              \
  do {                                                                                           \
    int _rc = (call);                                                                            \
    TORCH_CHECK(_rc == 0, "mxllm kernel launch failed (" #call ") rc=", _rc, " ",                 \
                hipGetErrorString((hipError_t)(_rc > 0 ? _rc : 1)));                             \
  } while (0)

inline const uint16_t* bf(const at::Tensor& t) {
  return reinterpret_cast<const uint16_t*>(t.data_ptr());
}
inline uint16_t* bfm(at::Tensor& t) { return reinterpret_cast<uint16_t*>(t.data_ptr()); }

void check_bf16(const at::Tensor& t, const char* name) {
  MX_CHECK(t.is_cuda(), name, " must be a GPU tensor");
  MX_CHECK(t.scalar_type() == at::kBFloat16, name, " must be bfloat16");
  MX_CHECK(t.is_contiguous(), name, " must be contiguous");
}
// a 2-D row-strided bf16 view (rows may be the left part of a wider buffer)
int64_t check_rows_bf16(const at::Tensor& t, const char* name) {
  MX_CHECK(t.is_cuda(), name, " must be a GPU tensor");
  MX_CHECK(t.scalar_type() == at::kBFloat16, name, " must be bfloat16");
  MX_CHECK(t.dim() == 2 && t.stride(1) == 1 && t.stride(0) >= t.size(1) && t.stride(0) % 8 == 0, name,
           " must be a row-major [T, H] view with a row stride that is a multiple of 8");
  return t.stride(0);
}
// [T, H] output whose rows live in a [T, H + pad] buffer (pad extra columns left to the caller)
at::Tensor empty_rows(int64_t T, int64_t H, int64_t pad, const at::TensorOptions& o) {
  if (pad <= 0) return at::empty({T, H}, o);
  return at::empty({T, H + pad}, o).narrow(1, 0, H);
}
void check_f32(const at::Tensor& t, const char* name) {
  MX_CHECK(t.is_cuda(), name, " must be a GPU tensor");
  MX_CHECK(t.scalar_type() == at::kFloat, name, " must be float32");
  MX_CHECK(t.is_contiguous(), name, " must be contiguous");
}

// Paged KV caches: k_cache/v_cache [blocks, Hkv, block, D] + block_table int32 [slots, maxb]
// (token p of slot s in block block_table[s][p / block]); without a block table the caches
// are [slots, Hkv, max_seq, D].
struct KvPages {
  const int32_t* bt = nullptr;
  int maxb = 0;
};
static KvPages kv_pages(const c10::optional<at::Tensor>& block_table, const at::Tensor& k_cache) {
  KvPages pg;
  if (block_table.has_value() && block_table->defined()) {
    const at::Tensor& t = *block_table;
    MX_CHECK(t.is_cuda() && t.scalar_type() == at::kInt && t.dim() == 2 && t.is_contiguous(),
             "block_table int32 [slots, max_blocks] contiguous GPU");
    MX_CHECK(k_cache.size(2) % 256 == 0, "paged KV: the block size must be a multiple of 256 tokens");
    pg.bt = t.data_ptr<int32_t>();
    pg.maxb = (int)t.size(1);
  }
  return pg;
}

// qkv [B, NH*D]; k_cache/v_cache [slots, Hkv, max_seq, D] (or paged); pos/slots int32 [B]

}  // namespace
