// Gated activations over row-strided GEMM outputs (gfx950).
//
//   clamped_glu: g = min(gate, limit), u = clamp(up, +-limit);
//                g * sigmoid(alpha (g + cubic g^3)) * (u + offset)
//   gelu_gate:   gelu_tanh(s) * table[token, offset + i]
//   side_gate:   x + y, then gelu_gate of (gate x): for few tokens, where two
//                elementwise launches and a GEMM of one narrow tile cost more than
//                reading the small weight once per token from L2
#include "common_t.h"
#include "gated_act.h"

template <typename T, int V>
__global__ __launch_bounds__(256) void clamped_glu_kernel(
    T* __restrict__ out, const T* __restrict__ gate_up, const float limit,
    const float alpha, const float offset, const float cubic, const int rows, const int inter,
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
    for (int k = 0; k < V; ++k) g[k] = clamped_glu_f(g[k], u[k], limit, alpha, offset, cubic);
    store_f<V>(out + r * out_stride + c, g);
  }
}

DEV float gelu_tanh_f(float z) {
  return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

// Workgroups (token, part of the outputs); the new residual row waits in LDS, in
// the GEMM's input precision, for its dot products.  Every part sums the row, one
// writes it: to a new residual, since the others may still be reading the old.
// All its loads are issued far ahead of their use: one token's latency is the cost.
template <typename T, int V>
__global__ __launch_bounds__(512) void side_gate_kernel(
    float* __restrict__ x_out, const float* __restrict__ x, const T* __restrict__ y,
    const T* __restrict__ gate, const int64_t* __restrict__ token_ids,
    const T* __restrict__ table, T* __restrict__ s, const int w, const int dim,
    const int64_t table_stride) {
  extern __shared__ char lds_raw[];
  T* row = (T*)lds_raw;
  const int64_t n = blockIdx.x;
  const int lane = threadIdx.x & 63;
  // a wave's two outputs; lane j keeps output j's table entry
  const int o0 = (blockIdx.y * 8 + (threadIdx.x >> 6)) * 2;
  const int oj = o0 + (lane & 1);
  const float e = oj < dim ? to_f(table[token_ids[n] * table_stride + oj]) : 0.f;
#pragma unroll 4
  for (int i = threadIdx.x * 4; i < w; i += 2048) {
    float a[4], b[4];
    load_f<4>(a, x + n * w + i);
    load_f<4>(b, y + n * w + i);
#pragma unroll
    for (int k = 0; k < 4; ++k) a[k] += b[k];
    if (blockIdx.y == 0) store_f<4>(x_out + n * w + i, a);
    store_f<4>(row + i, a);
  }
  __syncthreads();
  if (o0 >= dim) return;
  const T* g0 = gate + (int64_t)o0 * w;
  const T* g1 = gate + (int64_t)min(o0 + 1, dim - 1) * w;
  float acc0 = 0.f, acc1 = 0.f;
#pragma unroll 8
  for (int i = lane * V; i < w; i += 64 * V) {
    float v[V], p[V], q[V];
    load_f<V>(p, g0 + i);
    load_f<V>(q, g1 + i);
    load_f<V>(v, row + i);
#pragma unroll
    for (int k = 0; k < V; ++k) {
      acc0 += p[k] * v[k];
      acc1 += q[k] * v[k];
    }
  }
  acc0 = wave_sum(acc0);
  acc1 = wave_sum(acc1);
  // the product is an activation: model precision, as a GEMM would store it
  const float z = to_f(from_f<T>(lane & 1 ? acc1 : acc0));
  if (lane < 2 && oj < dim) s[n * dim + oj] = from_f<T>(gelu_tanh_f(z) * e);
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
  s[i] = from_f<T>(gelu_tanh_f(to_f(s[i])) * e);
}

extern "C" {

void launch_clamped_glu(bool bf16, void* out, const void* gate_up, float limit,
                        float alpha, float offset, float cubic, int rows, int inter,
                        int64_t in_stride, int64_t out_stride, hipStream_t stream) {
  const int v = bf16 ? 8 : 4;
  const int64_t want = ((int64_t)rows * (inter / v) + 255) / 256;
  const int grid = (int)(want < 4096 ? want : 4096);
  if (bf16)
    clamped_glu_kernel<bf16_t, 8><<<grid, 256, 0, stream>>>(
        (bf16_t*)out, (const bf16_t*)gate_up, limit, alpha, offset, cubic, rows, inter,
        in_stride, out_stride);
  else
    clamped_glu_kernel<float, 4><<<grid, 256, 0, stream>>>(
        (float*)out, (const float*)gate_up, limit, alpha, offset, cubic, rows, inter,
        in_stride, out_stride);
}

void launch_side_gate(bool bf16, float* x_out, const float* x, const void* y, const void* gate,
                      const int64_t* token_ids, const void* table, void* s, int n, int w,
                      int dim, int64_t table_stride, hipStream_t stream) {
  const dim3 grid(n, (dim + 15) / 16);
  if (bf16)
    side_gate_kernel<bf16_t, 8><<<grid, 512, w * 2, stream>>>(
        x_out, x, (const bf16_t*)y, (const bf16_t*)gate, token_ids, (const bf16_t*)table,
        (bf16_t*)s, w, dim, table_stride);
  else
    side_gate_kernel<float, 4><<<grid, 512, w * 4, stream>>>(
        x_out, x, (const float*)y, (const float*)gate, token_ids, (const float*)table, (float*)s, w,
        dim, table_stride);
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
