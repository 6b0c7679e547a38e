// Kernels built for both model dtypes (bf16 and fp32): element access and
// 16-byte vectors.  Math is fp32 either way.
#pragma once
#include "common.h"

DEV float to_f(bf16_t v) { return bf2f(v); }
DEV float to_f(float v) { return v; }
template <typename T> DEV T from_f(float v);
template <> DEV bf16_t from_f<bf16_t>(float v) {
  return __builtin_bit_cast(bf16_t, (__bf16)v);  // v_cvt_pk_bf16_f32
}
template <> DEV float from_f<float>(float v) { return v; }

// N consecutive elements <-> fp32; N * sizeof(T) is the access width and p is
// aligned to it
template <typename T, int N>
struct alignas(N * sizeof(T)) Pack {
  T v[N];
};

template <int N, typename T>
DEV void load_f(float* dst, const T* p) {
  const Pack<T, N> k = *(const Pack<T, N>*)p;
#pragma unroll
  for (int i = 0; i < N; ++i) dst[i] = to_f(k.v[i]);
}

template <int N, typename T>
DEV void store_f(T* p, const float* src) {
  Pack<T, N> k;
#pragma unroll
  for (int i = 0; i < N; ++i) k.v[i] = from_f<T>(src[i]);
  *(Pack<T, N>*)p = k;
}

DEV float sigmoid_f(float x) { return 1.f / (1.f + __expf(-x)); }
