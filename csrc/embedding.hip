// The two ends of a model with an fp32 residual (gfx950): scaled token embedding plus
// sinusoidal positions, and capped logits.
#include "common_t.h"

// grid (tokens, parts of the row).  cos_sin [2, P, half], half = ceil(w / 2): entry 2i gets the
// sine, 2i + 1 the cosine of angle i.
template <typename T, int V>
__global__ __launch_bounds__(256) void embed_positions_kernel(
    float* __restrict__ x, float* __restrict__ copy, const int64_t* __restrict__ token_ids,
    const int64_t* __restrict__ positions, const T* __restrict__ table,
    const float* __restrict__ cos_sin, const float scale, const int w, const int64_t vocab,
    const int64_t P) {
  const int64_t n = blockIdx.x;
  const int64_t tok = min(max(token_ids[n], (int64_t)0), vocab - 1);
  const int64_t p = min(max(positions[n], (int64_t)0), P - 1);
  const int half = (w + 1) >> 1;
  for (int i = (blockIdx.y * 256 + threadIdx.x) * V; i < w; i += gridDim.y * 256 * V) {
    float v[V];
    load_f<V>(v, table + tok * w + i);
#pragma unroll
    for (int k = 0; k < V; ++k) v[k] *= scale;
    if (cos_sin) {
#pragma unroll
      for (int k = 0; k < V; ++k)
        v[k] += cos_sin[((i + k) & 1 ? p : P + p) * half + ((i + k) >> 1)];
    }
    store_f<V>(x + n * w + i, v);
    if (copy) store_f<V>(copy + n * w + i, v);
  }
}

// cap tanh(x / cap) = cap - 2 cap / (e^(2 x / cap) + 1)
template <typename T, int V>
__global__ __launch_bounds__(256) void softcap_kernel(
    float* __restrict__ out, const T* __restrict__ x, const float cap, const int64_t n) {
  const int64_t step = (int64_t)gridDim.x * 256 * V;
  const float f = 2.f / cap;
  for (int64_t i = ((int64_t)blockIdx.x * 256 + threadIdx.x) * V; i < n; i += step) {
    float t[V];
    load_f<V>(t, x + i);
#pragma unroll
    for (int k = 0; k < V; ++k)
      t[k] = cap - 2.f * cap * __builtin_amdgcn_rcpf(__expf(t[k] * f) + 1.f);
    store_f<V>(out + i, t);
  }
}

extern "C" {

void launch_embed_positions(bool bf16, float* x, float* copy, const int64_t* token_ids,
                            const int64_t* positions, const void* table, const float* cos_sin,
                            float scale, int n, int w, int64_t vocab, int64_t P, hipStream_t stream) {
  const int v = w % 4 == 0 ? 4 : 1;
  const dim3 grid(n, (w / v + 255) / 256);
  if (bf16) {
    auto k = v == 4 ? embed_positions_kernel<bf16_t, 4> : embed_positions_kernel<bf16_t, 1>;
    k<<<grid, 256, 0, stream>>>(x, copy, token_ids, positions, (const bf16_t*)table, cos_sin, scale, w,
                                vocab, P);
  } else {
    auto k = v == 4 ? embed_positions_kernel<float, 4> : embed_positions_kernel<float, 1>;
    k<<<grid, 256, 0, stream>>>(x, copy, token_ids, positions, (const float*)table, cos_sin, scale, w,
                                vocab, P);
  }
}

void launch_softcap(bool bf16, float* out, const void* x, float cap, int64_t n,
                    hipStream_t stream) {
  const int v = n % 4 == 0 ? 4 : 1;
  const int64_t want = (n / v + 255) / 256;
  const int grid = (int)(want < 8192 ? want : 8192);
  if (bf16) {
    auto k = v == 4 ? softcap_kernel<bf16_t, 4> : softcap_kernel<bf16_t, 1>;
    k<<<grid, 256, 0, stream>>>(out, (const bf16_t*)x, cap, n);
  } else {
    auto k = v == 4 ? softcap_kernel<float, 4> : softcap_kernel<float, 1>;
    k<<<grid, 256, 0, stream>>>(out, (const float*)x, cap, n);
  }
}

}  // extern "C"
