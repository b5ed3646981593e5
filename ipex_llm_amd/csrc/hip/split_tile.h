// Pieces of the small matrix-core products whose f32 inputs must not be rounded
// (gates and decays of the recurrent mixers): with 16-bit weights an f32 value is
// split into three 16-bit parts whose sum it is.
#pragma once
#include <hip/hip_runtime.h>

namespace illm {
namespace sx {
namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

template <typename E> struct Parts { static constexpr int N = 1; };
template <> struct Parts<__bf16> { static constexpr int N = 3; };

// 8 consecutive weights of a row from index kk on, zeros from n on (vec: n is a multiple of 8, rows are 16-byte aligned)
template <typename E> struct Frag {
  E __attribute__((aligned(16))) v[8];
  __device__ __forceinline__ void load(const E* w, int kk, int n, bool vec) {
    if (vec && kk < n) {
      const uint4* s = (const uint4*)(w + kk);
      uint4* d = (uint4*)v;
#pragma unroll
      for (int i = 0; i < (int)(8 * sizeof(E) / 16); i++) d[i] = s[i];
    } else {
#pragma unroll
      for (int j = 0; j < 8; j++) v[j] = kk + j < n ? w[kk + j] : (E)0.f;
    }
  }
  __device__ __forceinline__ bf16x8 v8() const { return *(const bf16x8*)v; }
};

// an f32 value as the parts of E whose sum it is
template <int N> __device__ __forceinline__ void stage(float (*us)[N], int at, float v) { us[0][at] = v; }
template <int N> __device__ __forceinline__ void stage(__bf16 (*us)[N], int at, float v) {
  const __bf16 hi = (__bf16)v;
  const float r1 = v - (float)hi;
  const __bf16 mid = (__bf16)r1;
  us[0][at] = hi;
  us[1][at] = mid;
  us[2][at] = (__bf16)(r1 - (float)mid);
}

}  // namespace
}  // namespace sx
}  // namespace illm
