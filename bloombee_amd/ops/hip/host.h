// Host-side helpers of the torch bindings: checks, type dispatch, launches.
#pragma once

#include <torch/extension.h>
#include <c10/hip/HIPStream.h>
#include <hip/hip_runtime.h>

#include "rows.hip"

using torch::Tensor;
using OptTensor = c10::optional<Tensor>;
typedef unsigned short bf16_bits;

static hipStream_t cur_stream() {
  return c10::hip::getCurrentHIPStream().stream();
}

#define CHECK_T(x, st)                                                        \
  TORCH_CHECK((x).is_cuda() && (x).is_contiguous() &&                         \
                  (x).scalar_type() == (st),                                  \
              #x " must be a contiguous device tensor of ", toString(st))
#define CHECK_I32(x) CHECK_T(x, at::kInt)
#define CHECK_F32(x) CHECK_T(x, at::kFloat)

static void check_launch() {
  const hipError_t e = hipGetLastError();
  TORCH_CHECK(e == hipSuccess, "kernel launch: ", hipGetErrorString(e));
}

static void check_act(const Tensor& t) {
  TORCH_CHECK(t.is_cuda() && (t.scalar_type() == at::kBFloat16 ||
                              t.scalar_type() == at::kFloat),
              "activations must be bf16 or f32 on the device");
}

// f(element tag) with unsigned short for bf16, float for f32.
template <typename F>
static void by_type(at::ScalarType st, F f) {
  if (st == at::kBFloat16) f((bf16_bits)0);
  else f(0.f);
}

template <typename F>
static void by_bool(bool b, F f) {
  if (b) f(std::true_type{});
  else f(std::false_type{});
}

template <typename K>
static void allow_lds(K kernel, size_t bytes) {
  TORCH_CHECK(bytes <= 160 * 1024, "row too long for LDS: ", bytes, " bytes");
  if (bytes > 64 * 1024)
    TORCH_CHECK(hipFuncSetAttribute(
                    reinterpret_cast<const void*>(kernel),
                    hipFuncAttributeMaxDynamicSharedMemorySize,
                    (int)bytes) == hipSuccess,
                "cannot reserve ", bytes, " bytes of LDS");
}

static inline Parts as_parts(const Tensor& t) {
  check_act(t);
  TORCH_CHECK(t.dim() == 3 && t.is_contiguous());
  return Parts{t.data_ptr(), t.size(1) * t.size(2), (int)t.size(0),
               (int)t.size(2)};
}

// Keys a row sees at most.
template <typename Args>
static long seen_keys(const Args& a, long max_ctx) {
  long n = max_ctx;
  if (a.window > 0) n = std::min<long>(n, a.window);
  if (a.chunk > 0) n = std::min<long>(n, a.chunk);
  return n;
}

static inline bool all_of_8(std::initializer_list<long> v) {
  for (long x : v)
    if (x % 8) return false;
  return true;
}
