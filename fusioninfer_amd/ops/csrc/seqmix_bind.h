// Helpers shared by the binding units of _C_seqmix: operand checks, the
// activation-type dispatch, the current stream.
#pragma once

#include <torch/extension.h>

#include <c10/hip/HIPStream.h>
#include <hip/hip_runtime.h>

#include "seqmix.h"

namespace fi_bind {

using fi::u16;

inline hipStream_t stream() { return c10::hip::getCurrentHIPStream().stream(); }

inline bool is_act(const at::Tensor& t) {
  return t.scalar_type() == at::kFloat || t.scalar_type() == at::kBFloat16;
}

#define CHECK_ACT(t)                                                 \
  TORCH_CHECK((t).is_cuda(), #t " must be on the GPU");              \
  TORCH_CHECK(is_act(t), #t " must be float32 or bfloat16")
#define CHECK_F32(t)                                                  \
  TORCH_CHECK((t).is_cuda() && (t).scalar_type() == at::kFloat &&     \
                  (t).is_contiguous(),                                \
              #t " must be a contiguous float32 GPU tensor")
#define CHECK_I32(t)                                                  \
  TORCH_CHECK((t).is_cuda() && (t).scalar_type() == at::kInt &&       \
                  (t).is_contiguous(),                                \
              #t " must be a contiguous int32 GPU tensor")

// rows of a 2-D activation view whose last dim is dense
inline void check_rows(const at::Tensor& t, int64_t T, int64_t n, const char* what) {
  TORCH_CHECK(t.dim() == 2 && t.size(0) == T && t.size(1) == n &&
                  (t.stride(1) == 1 || n == 1),
              what, ": expected [", T, ", ", n, "] with dense rows");
}

inline void check_groups(const at::Tensor& seq_cu, const at::Tensor& seq_slots,
                  const at::Tensor& positions, int64_t T) {
  CHECK_I32(seq_cu);
  CHECK_I32(seq_slots);
  CHECK_I32(positions);
  TORCH_CHECK(seq_cu.numel() == seq_slots.numel() + 1);
  TORCH_CHECK(positions.numel() == T);
}

#define DISPATCH_ACT(t, ...)                          \
  if ((t).scalar_type() == at::kFloat) {              \
    using A = float;                                  \
    __VA_ARGS__;                                      \
  } else {                                            \
    using A = u16;                                    \
    __VA_ARGS__;                                      \
  }

template <typename A>
A* ptr(const at::Tensor& t) {
  return reinterpret_cast<A*>(t.data_ptr());
}

}  // namespace fi_bind

// bindings that live in units of their own (seqmix_hyper_bindings.hip,
// seqmix_scan_bindings.hip)
void register_hyper_ops(pybind11::module& m);
void register_scan_ops(pybind11::module& m);
