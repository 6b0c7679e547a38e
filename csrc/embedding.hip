// The two ends of a model with an fp32 residual (gfx950): token embedding plus
// sinusoidal positions, and capped logits.
#include "common_t.h"

// A workgroup per token.  cos_sin [2, P, half], half = ceil(w / 2): entry 2i gets the
// sine, 2i + 1 the cosine of angle i.
template <typename T>
__global__ __launch_bounds__(256) void embed_positions_kernel(
    float* __restrict__ x, float* __restrict__ copy, const int64_t* __restrict__ token_ids,
    const int64_t* __restrict__ positions, const T* __restrict__ table,
    const float* __restrict__ cos_sin, const int w, const int64_t vocab, const int64_t P) {
  const int64_t n = blockIdx.x;
  const int64_t tok = min(max(token_ids[n], (int64_t)0), vocab - 1);
  const int64_t p = min(max(positions[n], (int64_t)0), P - 1);
  const int half = (w + 1) >> 1;
  for (int i = threadIdx.x; i < w; i += 256) {
    float v = to_f(table[tok * w + i]);
    if (cos_sin) v += cos_sin[((i & 1 ? 0 : P) + p) * half + (i >> 1)];
    x[n * w + i] = v;
    if (copy) copy[n * w + i] = v;
  }
}

template <typename T>
__global__ __launch_bounds__(256) void softcap_kernel(
    float* __restrict__ out, const T* __restrict__ x, const float cap, const int64_t n) {
  const int64_t step = (int64_t)gridDim.x * 256;
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += step)
    out[i] = cap * tanhf(to_f(x[i]) / cap);
}

extern "C" {

void launch_embed_positions(bool bf16, float* x, float* copy, const int64_t* token_ids,
                            const int64_t* positions, const void* table, const float* cos_sin,
                            int n, int w, int64_t vocab, int64_t P, hipStream_t stream) {
  if (bf16)
    embed_positions_kernel<bf16_t><<<n, 256, 0, stream>>>(
        x, copy, token_ids, positions, (const bf16_t*)table, cos_sin, w, vocab, P);
  else
    embed_positions_kernel<float><<<n, 256, 0, stream>>>(
        x, copy, token_ids, positions, (const float*)table, cos_sin, w, vocab, P);
}

void launch_softcap(bool bf16, float* out, const void* x, float cap, int64_t n,
                    hipStream_t stream) {
  const int64_t want = (n + 255) / 256;
  const int grid = (int)(want < 8192 ? want : 8192);
  if (bf16)
    softcap_kernel<bf16_t><<<grid, 256, 0, stream>>>(out, (const bf16_t*)x, cap, n);
  else
    softcap_kernel<float><<<grid, 256, 0, stream>>>(out, (const float*)x, cap, n);
}

}  // extern "C"
