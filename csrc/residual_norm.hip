// Norms around an fp32 residual stream (gfx950).
//
// residual_norm is one pass over a row: optionally add mult * y, or mult *
// rmsnorm(y) * w_y, to the residual, optionally file the result as the newest depth
// state and replace it by a weighted sum of all states, then emit norm(x) * w_x (layer
// or RMS norm) or x itself for the next GEMM.  What is added may include a weighted sum
// of several rows (chosen experts' results) and be gated; the norm may be written a second
// time under another weight.  The row lives in LDS between the reductions (each thread re-reads only what
// it wrote, so the row itself needs no barrier).  Mean first, then the squared
// deviations: no cancellation.
#include "common_t.h"
#include "residual_norm.h"

// The depth average would read every state once per layer.  In blocks of
// DEPTH_AHEAD + 1 layers, the first one reads them all, for itself and for the others,
// which then read their partial sum and the few states made since.
template <int V>
DEV void depth_average(float* t, const NormForm& f, const int64_t at) {
  const int last = f.n_states - 1;
  store_f<V>(f.states + last * f.plane + at, t);
  float sum[V];
#pragma unroll
  for (int k = 0; k < V; ++k) sum[k] = f.coef[last] * t[k];
  if (f.first > 0) {
    float s[V];
    load_f<V>(s, f.partial + f.ready * f.plane + at);
#pragma unroll
    for (int k = 0; k < V; ++k) sum[k] += s[k];
    for (int j = f.first; j < last; ++j) {
      load_f<V>(s, f.states + j * f.plane + at);
#pragma unroll
      for (int k = 0; k < V; ++k) sum[k] += f.coef[j] * s[k];
    }
  } else {
    const float* c[DEPTH_AHEAD];
    float p[DEPTH_AHEAD][V];
#pragma unroll
    for (int a = 0; a < DEPTH_AHEAD; ++a) {
      c[a] = f.coef + (a < f.ahead ? (a + 1) * f.coef_stride : 0);
#pragma unroll
      for (int k = 0; k < V; ++k) p[a][k] = c[a][last] * t[k];
    }
#pragma unroll 8
    for (int j = 0; j < last; ++j) {
      float s[V];
      load_f<V>(s, f.states + j * f.plane + at);
#pragma unroll
      for (int k = 0; k < V; ++k) {
        sum[k] += f.coef[j] * s[k];
#pragma unroll
        for (int a = 0; a < DEPTH_AHEAD; ++a) p[a][k] += c[a][j] * s[k];
      }
    }
#pragma unroll
    for (int a = 0; a < DEPTH_AHEAD; ++a)
      if (a < f.ahead) store_f<V>(f.partial + a * f.plane + at, p[a]);
  }
#pragma unroll
  for (int k = 0; k < V; ++k) t[k] = sum[k];
}

// what is added to x at i: y, the experts' rows and the gate
template <typename T, int V>
DEV void addend(float* d, const T* y, const NormForm& f, const int w, const int i) {
  load_f<V>(d, y + (int64_t)blockIdx.x * w + i);
  const T* er = (const T*)f.rows + (int64_t)blockIdx.x * f.top * w + i;
  const float* ew = f.weights + (int64_t)blockIdx.x * f.top;
#pragma unroll 4
  for (int j = 0; j < f.top; ++j) {
    float e[V];
    load_f<V>(e, er + (int64_t)j * w);
#pragma unroll
    for (int k = 0; k < V; ++k) d[k] += ew[j] * e[k];
  }
  if (f.gate) {
    float g[V];
    load_f<V>(g, (const T*)f.gate + (int64_t)blockIdx.x * f.gate_stride + i);
#pragma unroll
    for (int k = 0; k < V; ++k) d[k] *= sigmoid_f(g[k]);
  }
}

template <typename T, int V, bool DEPTH>
__global__ __launch_bounds__(1024) void residual_norm_kernel(
    float* __restrict__ x,            // [n, w], updated if y
    const T* __restrict__ y,          // [n, w] or null
    const T* __restrict__ y_norm,     // [w] or null: plain add
    const T* __restrict__ x_norm,     // [w] or null: out = x
    T* __restrict__ out,              // [n, w] rows out_stride apart, or null
    const float eps, const int w, const int64_t out_stride, const NormForm f) {
  extern __shared__ float row[];
  __shared__ float scratch[3][16];
  float* xr = x + (int64_t)blockIdx.x * w;
  const int step = blockDim.x * V;
  const int i0 = threadIdx.x * V;

  float y_scale = 1.f;
  if (y && y_norm) {
    float ss = 0.f;
    for (int i = i0; i < w; i += step) {
      float t[V];
      addend<T, V>(t, y, f, w, i);
#pragma unroll
      for (int k = 0; k < V; ++k) {
        ss += t[k] * t[k];
        row[i + k] = t[k];
      }
    }
    y_scale = rsqrtf(block_sum(ss, scratch[0]) / w + eps);
  }
  float sum = 0.f;
  for (int i = i0; i < w; i += step) {
    float t[V];
    load_f<V>(t, xr + i);
    if (y) {
      float d[V];
      if (y_norm) {
        load_f<V>(d, y_norm + i);
#pragma unroll
        for (int k = 0; k < V; ++k) d[k] = (f.offset + d[k]) * row[i + k] * y_scale;
      } else {
        addend<T, V>(d, y, f, w, i);
      }
#pragma unroll
      for (int k = 0; k < V; ++k) t[k] += f.mult * d[k];
    }
    if (DEPTH) depth_average<V>(t, f, (int64_t)blockIdx.x * w + i);
    if (y || DEPTH) store_f<V>(xr + i, t);
#pragma unroll
    for (int k = 0; k < V; ++k) {
      sum += t[k];
      row[i + k] = t[k];
    }
  }
  if (!out) return;
  T* orow = out + (int64_t)blockIdx.x * out_stride;
  float mean = 0.f, inv = 1.f;
  if (x_norm) {
    if (f.center) mean = block_sum(sum, scratch[1]) / w;
    float ss = 0.f;
    for (int i = i0; i < w; i += step)
#pragma unroll
      for (int k = 0; k < V; ++k) {
        const float c = row[i + k] - mean;
        ss += c * c;
      }
    inv = rsqrtf(block_sum(ss, scratch[2]) / w + eps);
  }
  T* orow2 = f.out2 ? (T*)f.out2 + (int64_t)blockIdx.x * f.out2_stride : nullptr;
  for (int i = i0; i < w; i += step) {
    float t[V];
#pragma unroll
    for (int k = 0; k < V; ++k) t[k] = (row[i + k] - mean) * inv;
    if (orow2) {
      float g[V];
      load_f<V>(g, (const T*)f.x_norm2 + i);
#pragma unroll
      for (int k = 0; k < V; ++k) g[k] = (f.offset + g[k]) * t[k];
      store_f<V>(orow2 + i, g);
    }
    if (x_norm) {
      float g[V];
      load_f<V>(g, x_norm + i);
#pragma unroll
      for (int k = 0; k < V; ++k) t[k] *= f.offset + g[k];
    }
    store_f<V>(orow + i, t);
  }
}

template <typename T, int V>
__global__ __launch_bounds__(256) void add_to_residual_kernel(
    float* __restrict__ x, const T* __restrict__ y, T* __restrict__ out,
    const int64_t n) {
  const int64_t step = (int64_t)gridDim.x * blockDim.x * V;
  for (int64_t i = ((int64_t)blockIdx.x * blockDim.x + threadIdx.x) * V; i < n; i += step) {
    float a[V], b[V];
    load_f<V>(a, x + i);
    load_f<V>(b, y + i);
#pragma unroll
    for (int k = 0; k < V; ++k) a[k] += b[k];
    store_f<V>(x + i, a);
    if (out) store_f<V>(out + i, a);
  }
}

template <typename T>
static void residual_norm_t(float* x, const void* y, const void* y_norm,
                            const void* x_norm, void* out, float eps, int n,
                            int w, int64_t out_stride, const NormForm& f,
                            hipStream_t stream) {
  const bool vec = w % 4 == 0 && out_stride % 4 == 0 && f.out2_stride % 4 == 0 &&
                   f.gate_stride % 4 == 0 && (uintptr_t)f.gate % (4 * sizeof(T)) == 0;
  int threads = w >= 1024 ? 256 : w >= 512 ? 128 : 64;
  // few rows: the latency of one counts
  while (n <= 512 && threads < 1024 && threads * 4 < w) threads *= 2;
  auto k = f.n_states ? (vec ? residual_norm_kernel<T, 4, true> : residual_norm_kernel<T, 1, true>)
                      : (vec ? residual_norm_kernel<T, 4, false> : residual_norm_kernel<T, 1, false>);
  k<<<n, threads, w * sizeof(float), stream>>>(
      x, (const T*)y, (const T*)y_norm, (const T*)x_norm, (T*)out, eps, w, out_stride, f);
}

extern "C" {

void launch_residual_norm(bool bf16, float* x, const void* y, const void* y_norm,
                          const void* x_norm, void* out, float eps, int n, int w,
                          int64_t out_stride, const NormForm* f, hipStream_t stream) {
  (bf16 ? residual_norm_t<bf16_t> : residual_norm_t<float>)(
      x, y, y_norm, x_norm, out, eps, n, w, out_stride, *f, stream);
}

void launch_add_to_residual(bool bf16, float* x, const void* y, void* out,
                            int64_t n, hipStream_t stream) {
  const int v = n % 4 == 0 ? 4 : 1;
  const int64_t want = (n / v + 255) / 256;
  const int grid = (int)(want < 4096 ? want : 4096);
  if (bf16) {
    auto k = v == 4 ? add_to_residual_kernel<bf16_t, 4> : add_to_residual_kernel<bf16_t, 1>;
    k<<<grid, 256, 0, stream>>>(x, (const bf16_t*)y, (bf16_t*)out, n);
  } else {
    auto k = v == 4 ? add_to_residual_kernel<float, 4> : add_to_residual_kernel<float, 1>;
    k<<<grid, 256, 0, stream>>>(x, (const float*)y, (float*)out, n);
  }
}

}  // extern "C"
