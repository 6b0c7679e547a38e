// Gated activations over row-strided GEMM outputs (gfx950).
//
//   clamped_glu: g = min(gate, limit), u = clamp(up, +-limit);
//                g * sigmoid(alpha g) * (u + offset)
//   gelu_gate:   gelu_tanh(s) * table[token, offset + i]
#include "common_t.h"

template <typename T, int V>
__global__ __launch_bounds__(256) void clamped_glu_kernel(
    T* __restrict__ out, const T* __restrict__ gate_up, const float limit,
    const float alpha, const float offset, const int rows, const int inter,
    const int64_t in_stride, const int64_t out_stride) {
  const int per_row = inter / V;
  const int64_t total = (int64_t)rows * per_row;
  const int64_t step = (int64_t)gridDim.x * blockDim.x;
  for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += step) {
    const int64_t r = i / per_row;
    const int c = (int)(i - r * per_row) * V;
    float g[V], u[V];
    load_f<V>(g, gate_up + r * in_stride + c);
    load_f<V>(u, gate_up + r * in_stride + inter + c);
#pragma unroll
    for (int k = 0; k < V; ++k) {
      const float gc = fminf(g[k], limit);
      const float uc = fminf(fmaxf(u[k], -limit), limit);
      g[k] = gc * sigmoid_f(alpha * gc) * (uc + offset);
    }
    store_f<V>(out + r * out_stride + c, g);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void gelu_gate_kernel(
    T* __restrict__ s, const int64_t* __restrict__ token_ids,
    const T* __restrict__ table, const int dim, const int64_t total,
    const int64_t table_stride) {
  const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= total) return;
  const int64_t r = i / dim;
  const float e = to_f(table[token_ids[r] * table_stride + (i - r * dim)]);
  const float z = to_f(s[i]);
  const float t = tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z));
  s[i] = from_f<T>(0.5f * z * (1.f + t) * e);
}

extern "C" {

void launch_clamped_glu(bool bf16, void* out, const void* gate_up, float limit,
                        float alpha, float offset, int rows, int inter,
                        int64_t in_stride, int64_t out_stride, hipStream_t stream) {
  const int v = bf16 ? 8 : 4;
  const int64_t want = ((int64_t)rows * (inter / v) + 255) / 256;
  const int grid = (int)(want < 4096 ? want : 4096);
  if (bf16)
    clamped_glu_kernel<bf16_t, 8><<<grid, 256, 0, stream>>>(
        (bf16_t*)out, (const bf16_t*)gate_up, limit, alpha, offset, rows, inter,
        in_stride, out_stride);
  else
    clamped_glu_kernel<float, 4><<<grid, 256, 0, stream>>>(
        (float*)out, (const float*)gate_up, limit, alpha, offset, rows, inter,
        in_stride, out_stride);
}

void launch_gelu_gate(bool bf16, void* s, const int64_t* token_ids, const void* table,
                      int rows, int dim, int64_t table_stride, hipStream_t stream) {
  const int64_t total = (int64_t)rows * dim;
  const int grid = (int)((total + 255) / 256);
  if (bf16)
    gelu_gate_kernel<bf16_t><<<grid, 256, 0, stream>>>(
        (bf16_t*)s, token_ids, (const bf16_t*)table, dim, total, table_stride);
  else
    gelu_gate_kernel<float><<<grid, 256, 0, stream>>>(
        (float*)s, token_ids, (const float*)table, dim, total, table_stride);
}

}  // extern "C"
