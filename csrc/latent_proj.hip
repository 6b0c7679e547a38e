// Per-token kernels around latent attention (gfx950): its normed inputs with the
// cache-row write, and the per-head products that absorb the key and value up-projections.
//
// Rotations here pair dimension 2i with 2i+1; cos_sin is [2, P, rot_dim/2] fp32.
#include "common_t.h"

typedef __bf16 bf16x8_v __attribute__((ext_vector_type(8)));
typedef float f32x4_v __attribute__((ext_vector_type(4)));

// A wave per token and job.  Job 0: RMS-norm kv[:kv_rank], rotate kv[kv_rank:],
// write the padded cache row [kv_rank -> rank | rot_dim -> row - rank] at its slot.
// Job 1 (low-rank queries): cq = rmsnorm(q) over the first q_rank of its k columns.
template <typename T, int V>
__global__ __launch_bounds__(256) void latent_inputs_kernel(
    T* __restrict__ cache, const T* __restrict__ kv, const T* __restrict__ norm_w,
    const int64_t* __restrict__ positions, const int64_t* __restrict__ slots,
    const float* __restrict__ cos_sin, const float eps, const int N,
    const int kv_rank, const int rot_dim, const int rank, const int row,
    const int64_t kv_stride, const int64_t P, T* __restrict__ cq,
    const T* __restrict__ q, const T* __restrict__ q_norm, const int k,
    const int q_rank, const int64_t q_stride) {
  const int n = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (n >= N) return;
  const int lane = threadIdx.x & 63;
  if (blockIdx.y == 1) {
    const T* src = q + n * q_stride;
    float ss = 0.f;
    for (int i = lane * V; i < k; i += 64 * V) {
      float t[V];
      load_f<V>(t, src + i);  // columns q_rank.. are zero
#pragma unroll
      for (int j = 0; j < V; ++j) ss += t[j] * t[j];
    }
    const float inv = rsqrtf(wave_sum(ss) / q_rank + eps);
    for (int i = lane * V; i < k; i += 64 * V) {
      float t[V], w[V];
      load_f<V>(t, src + i);
      load_f<V>(w, q_norm + i);
#pragma unroll
      for (int j = 0; j < V; ++j) t[j] *= inv * w[j];
      store_f<V>(cq + (int64_t)n * k + i, t);
    }
    return;
  }
  const T* src = kv + n * kv_stride;
  T* dst = cache + slots[n] * row;
  const int half = rot_dim >> 1;
  const float* ct = cos_sin + positions[n] * half;
  const float* st = ct + P * half;
  for (int i = lane; 2 * i < row - rank; i += 64) {
    float u = 0.f, v = 0.f;
    if (i < half) {
      const float a = to_f(src[kv_rank + 2 * i]), b = to_f(src[kv_rank + 2 * i + 1]);
      u = a * ct[i] - b * st[i];
      v = b * ct[i] + a * st[i];
    }
    const float uv[2] = {u, v};
    store_f<2>(dst + rank + 2 * i, uv);
  }
  float ss = 0.f;
  const bool wide = kv_rank % (64 * V) == 0 &&
                    ((uintptr_t)kv | (uintptr_t)(kv_stride * sizeof(T))) % 16 == 0;
  if (wide) {
    for (int i = lane * V; i < kv_rank; i += 64 * V) {
      float t[V];
      load_f<V>(t, src + i);
#pragma unroll
      for (int j = 0; j < V; ++j) ss += t[j] * t[j];
    }
    const float inv = rsqrtf(wave_sum(ss) / kv_rank + eps);
    for (int i = lane * V; i < kv_rank; i += 64 * V) {
      float t[V], w[V];
      load_f<V>(t, src + i);
      load_f<V>(w, norm_w + i);
#pragma unroll
      for (int j = 0; j < V; ++j) t[j] *= inv * w[j];
      store_f<V>(dst + i, t);
    }
    for (int i = kv_rank + lane; i < rank; i += 64) dst[i] = from_f<T>(0.f);
    return;
  }
  for (int i = lane; i < kv_rank; i += 64) {
    const float f = to_f(src[i]);
    ss += f * f;
  }
  const float inv = rsqrtf(wave_sum(ss) / kv_rank + eps);
  for (int i = lane; i < rank; i += 64)
    dst[i] = from_f<T>(i < kv_rank ? to_f(src[i]) * inv * to_f(norm_w[i]) : 0.f);
}

// out[n, h, :O] = W[h] x[n, h, :K] (* sigmoid(gate[n, h])) on the matrix cores.
// A wave owns 16*OT outputs x 16*TT tokens; both operands are K-contiguous, so the
// fragments load straight from global memory (weights are small enough to stay
// in L2, tokens of one head in L1).  A = weights, B = tokens: a lane ends up
// with 4 consecutive outputs of one token.
template <int OT, int TT>
__global__ __launch_bounds__(256) void head_linear_mfma_kernel(
    bf16_t* __restrict__ out, const bf16_t* __restrict__ x,
    const bf16_t* __restrict__ w, const bf16_t* __restrict__ gate, const int N,
    const int O, const int K, const int64_t x_row, const int x_head,
    const int64_t out_row, const int out_head, const int64_t gate_row) {
  const int h = blockIdx.z;
  const int lane = threadIdx.x & 63;
  const int c = lane & 15, g = lane >> 4;
  const int o0 = (blockIdx.y * (blockDim.x >> 6) + (threadIdx.x >> 6)) * (16 * OT);
  if (o0 >= O) return;
  const int n0 = blockIdx.x * (16 * TT);
  const bf16_t* wp[OT];
  const bf16_t* xp[TT];
#pragma unroll
  for (int i = 0; i < OT; ++i)
    wp[i] = w + ((int64_t)h * O + min(o0 + i * 16 + c, O - 1)) * K + g * 8;
#pragma unroll
  for (int t = 0; t < TT; ++t)
    xp[t] = x + (int64_t)min(n0 + t * 16 + c, N - 1) * x_row + (int64_t)h * x_head + g * 8;
  f32x4_v acc[OT][TT] = {};
#pragma unroll 4
  for (int k = 0; k < K; k += 32) {
    bf16x8_v a[OT], b[TT];
#pragma unroll
    for (int i = 0; i < OT; ++i) a[i] = *(const bf16x8_v*)(wp[i] + k);
#pragma unroll
    for (int t = 0; t < TT; ++t) b[t] = *(const bf16x8_v*)(xp[t] + k);
#pragma unroll
    for (int i = 0; i < OT; ++i)
#pragma unroll
      for (int t = 0; t < TT; ++t)
        acc[i][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[i], b[t], acc[i][t], 0, 0, 0);
  }
#pragma unroll
  for (int t = 0; t < TT; ++t) {
    const int n = n0 + t * 16 + c;
    if (n >= N) continue;
    const float s = gate ? sigmoid_f(bf2f(gate[n * gate_row + h])) : 1.f;
    bf16_t* dst = out + n * out_row + (int64_t)h * out_head;
#pragma unroll
    for (int i = 0; i < OT; ++i) {
      const int o = o0 + i * 16 + g * 4;  // O is a multiple of 32
      if (o >= O) continue;
      const float v[4] = {acc[i][t][0] * s, acc[i][t][1] * s, acc[i][t][2] * s,
                          acc[i][t][3] * s};
      store_f<4>(dst + o, v);
    }
  }
}

// fp32 twin: a thread per output, 4 tokens per block in flight.
__global__ __launch_bounds__(256) void head_linear_f32_kernel(
    float* __restrict__ out, const float* __restrict__ x, const float* __restrict__ w,
    const float* __restrict__ gate, const int N, const int O, const int K,
    const int64_t x_row, const int x_head, const int64_t out_row,
    const int out_head, const int64_t gate_row) {
  const int h = blockIdx.z;
  const int o = blockIdx.y * 64 + (threadIdx.x & 63);
  const int n = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (o >= O || n >= N) return;
  const float* wr = w + ((int64_t)h * O + o) * K;
  const float* xr = x + n * x_row + (int64_t)h * x_head;
  float acc = 0.f;
  for (int k = 0; k < K; k += 4) {
    float a[4], b[4];
    load_f<4>(a, wr + k);
    load_f<4>(b, xr + k);
#pragma unroll
    for (int j = 0; j < 4; ++j) acc += a[j] * b[j];
  }
  if (gate) acc *= sigmoid_f(gate[n * gate_row + h]);
  out[n * out_row + (int64_t)h * out_head + o] = acc;
}

extern "C" {

void launch_latent_inputs(bool bf16, void* cache, const void* kv, const void* norm_w,
                          const int64_t* positions, const int64_t* slots,
                          const float* cos_sin, float eps, int N, int kv_rank, int rot_dim,
                          int rank, int row, int64_t kv_stride, int64_t P, void* cq,
                          const void* q, const void* q_norm, int k, int q_rank,
                          int64_t q_stride, hipStream_t stream) {
  const dim3 grid((N + 3) / 4, q ? 2 : 1);
  if (bf16)
    latent_inputs_kernel<bf16_t, 8><<<grid, 256, 0, stream>>>(
        (bf16_t*)cache, (const bf16_t*)kv, (const bf16_t*)norm_w, positions, slots,
        cos_sin, eps, N, kv_rank, rot_dim, rank, row, kv_stride, P, (bf16_t*)cq,
        (const bf16_t*)q, (const bf16_t*)q_norm, k, q_rank, q_stride);
  else
    latent_inputs_kernel<float, 4><<<grid, 256, 0, stream>>>(
        (float*)cache, (const float*)kv, (const float*)norm_w, positions, slots, cos_sin,
        eps, N, kv_rank, rot_dim, rank, row, kv_stride, P, (float*)cq, (const float*)q,
        (const float*)q_norm, k, q_rank, q_stride);
}

void launch_head_linear(bool bf16, void* out, const void* x, const void* w,
                        const void* gate, int N, int H, int O, int K, int64_t x_row,
                        int x_head, int64_t out_row, int out_head, int64_t gate_row,
                        hipStream_t stream) {
  if (!bf16) {
    dim3 grid((N + 3) / 4, (O + 63) / 64, H);
    head_linear_f32_kernel<<<grid, 256, 0, stream>>>(
        (float*)out, (const float*)x, (const float*)w, (const float*)gate, N, O, K,
        x_row, x_head, out_row, out_head, gate_row);
    return;
  }
  // few tokens: small wave tiles, so that enough waves hide the load latency
  const int tt = N > 2048 ? 4 : N > 256 ? 2 : 1;
  const int ot = tt == 1 ? 2 : 4;
  const int tiles = (O + 16 * ot - 1) / (16 * ot);
  const int waves = tiles < 4 ? tiles : 4;
  dim3 grid((N + 16 * tt - 1) / (16 * tt), (tiles + waves - 1) / waves, H);
  auto k = tt == 4 ? head_linear_mfma_kernel<4, 4>
                   : tt == 2 ? head_linear_mfma_kernel<4, 2> : head_linear_mfma_kernel<2, 1>;
  k<<<grid, 64 * waves, 0, stream>>>(
      (bf16_t*)out, (const bf16_t*)x, (const bf16_t*)w, (const bf16_t*)gate, N, O, K,
      x_row, x_head, out_row, out_head, gate_row);
}

}  // extern "C"
