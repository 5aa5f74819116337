// check.h — host-side checks shared by the bindings: every shape a kernel's
// indexing relies on is checked before its launch.
#pragma once
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>
#include <ATen/hip/impl/HIPStreamMasqueradingAsCUDA.h>

#include <hip/hip_runtime.h>

namespace {

using torch::Tensor;
using OptTensor = c10::optional<Tensor>;

inline hipStream_t cur_stream() {
  return at::hip::getCurrentHIPStreamMasqueradingAsCUDA().stream();
}

inline void check_hip(hipError_t e, const char* what) {
  TORCH_CHECK(e == hipSuccess, what, ": ", hipGetErrorString(e));
}

inline void check(const Tensor& t, at::ScalarType type, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.is_contiguous(), name,
              " must be contiguous on the GPU");
  TORCH_CHECK(t.scalar_type() == type, name, " has type ", t.scalar_type());
}

inline void sized(const Tensor& t, std::initializer_list<int64_t> want,
                  const char* name) {
  TORCH_CHECK(t.sizes() == at::IntArrayRef(want.begin(), want.size()), name,
              " has sizes ", t.sizes(), ", expected ",
              at::IntArrayRef(want.begin(), want.size()));
}

// bf16 or float activations
inline int act(const Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.is_contiguous(), name,
              " must be contiguous on the GPU");
  if (t.scalar_type() == at::kFloat) return 1;
  TORCH_CHECK(t.scalar_type() == at::kBFloat16, name,
              " must be bf16 or float");
  return 0;
}

inline void same_act(const Tensor& t, int f32, const char* name) {
  TORCH_CHECK(act(t, name) == f32, name, ": mixed activation types");
}

inline float* fp(const Tensor& t) { return t.data_ptr<float>(); }
inline int32_t* ip(const Tensor& t) { return t.data_ptr<int32_t>(); }

// rows [base, base + n) of a batch
inline void check_rows(const Tensor& positions, const Tensor& row_seq,
                       int64_t base, int64_t n) {
  check(positions, at::kInt, "positions");
  check(row_seq, at::kInt, "row_seq");
  TORCH_CHECK(base >= 0 && base + n <= positions.numel() &&
                  positions.numel() == row_seq.numel(), "batch rows");
}

}  // namespace

extern "C" hipError_t lds_attn_rows(
    int, const void* const*, const int64_t*, int, int, int, int, int, float,
    const int32_t*, const int32_t*, int, const int32_t*, int, int,
    const int32_t*, int, float, void*, int64_t, int64_t, int, int,
    hipStream_t);

// bindings of ops_grouped.hip
void bind_grouped(pybind11::module& m);
