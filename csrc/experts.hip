// Mixture of experts (gfx950): routing, grouping by expert, and the experts' products
// for few rows per expert and for fp32.  experts_gemm.hip has the product for many.
//
// Nothing here depends on the routing but memory contents: grids come from host values,
// so decode steps can be captured.
#include "experts.h"
#include "gated_act.h"

typedef __bf16 bf16x8_v __attribute__((ext_vector_type(8)));
typedef float f32x4_v __attribute__((ext_vector_type(4)));

#define ROUTE_T 16  // tokens per workgroup
#define AHEAD 8      // turns whose ids are loaded together

// The wave picks the ``top`` largest of logits[0 .. E) (overwritten), the lower index
// among equals, and their weights: scale times their softmax or, with ``scores``, times
// the chosen scores over their sum.
static DEV void choose(float* logits, const float* scores, int E, int top, float scale, int* ids,
                       float* weights) {
  const int lane = threadIdx.x & 63;
  float mine = -INFINITY, first = 0.f;
  int my_id = 0;
  for (int j = 0; j < top; ++j) {
    float best = -INFINITY;
    int at = 1 << 30;
    for (int e = lane; e < E; e += 64)
      if (logits[e] > best) {
        best = logits[e];
        at = e;
      }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) {
      const float v = __shfl_xor(best, off, 64);
      const int i = __shfl_xor(at, off, 64);
      if (v > best || (v == best && i < at)) {
        best = v;
        at = i;
      }
    }
    at = min(at, E - 1);  // whatever the logits are, an id stays an id
    if (j == 0) first = best;
    if (lane == j) {
      mine = scores ? scores[at] : best;
      my_id = at;
    }
    if (lane == (at & 63)) logits[at] = -INFINITY;
  }
  const float w = lane >= top ? 0.f : scores ? mine : expf(mine - first);
  const float sum = wave_sum(w) + (scores ? 1e-20f : 0.f);
  if (lane < top) {
    ids[lane] = my_id;
    weights[lane] = scale * w / sum;
  }
}

// 16 tokens a workgroup: its waves split K in blocks of 64, partial logits meet in LDS.
// NF fragments of 16 experts at a time.
// Dynamic LDS: [waves][16][E16] floats, E16 = E rounded up to 16.
template <int NF>
__global__ __launch_bounds__(1024) void route_mfma_kernel(
    int* __restrict__ ids, float* __restrict__ weights, const bf16_t* __restrict__ h,
    const bf16_t* __restrict__ w, const float* __restrict__ bias, const int N, const int E,
    const int K, const int top, const int64_t h_stride, const bool sigmoid, const float scale) {
  extern __shared__ float part[];
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, waves = blockDim.x >> 6;
  const int c = lane & 15, g = lane >> 4;
  const int E16 = (E + 15) & ~15, logits = ROUTE_T * E16;
  const int n0 = blockIdx.x * ROUTE_T;
  const bf16_t* hp = h + (int64_t)min(n0 + c, N - 1) * h_stride + g * 8;
  float* mine = part + (int64_t)wid * logits;
  for (int e0 = 0; e0 < E16; e0 += 16 * NF) {
    const bf16_t* wp[NF];
#pragma unroll
    for (int i = 0; i < NF; ++i)
      wp[i] = w + (int64_t)min(e0 + i * 16 + c, E - 1) * K + g * 8;
    f32x4_v acc[NF] = {};
#pragma unroll 4
    for (int k = wid * 64; k < K; k += waves * 64) {
#pragma unroll
      for (int s = 0; s < 64; s += 32) {
        const bf16x8_v b = *(const bf16x8_v*)(hp + k + s);
#pragma unroll
        for (int i = 0; i < NF; ++i) {
          const bf16x8_v f = *(const bf16x8_v*)(wp[i] + k + s);
          acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f, b, acc[i], 0, 0, 0);
        }
      }
    }
#pragma unroll
    for (int i = 0; i < NF; ++i) {
      const int e = e0 + i * 16 + g * 4;
      if (e < E16) *(f32x4_v*)(mine + c * E16 + e) = acc[i];
    }
  }
  __syncthreads();
  // the first wave's part becomes the logits, the second's the scores
  for (int i = threadIdx.x; i < logits; i += blockDim.x) {
    const int e = i % E16;
    float z = 0.f;
    for (int p = 0; p < waves; ++p) z += part[(int64_t)p * logits + i];
    if (sigmoid) part[logits + i] = z = 1.f / (1.f + expf(-z));
    part[i] = e < E ? z + (bias ? bias[e] : 0.f) : -INFINITY;
  }
  __syncthreads();
  for (int t = wid; t < min(ROUTE_T, N - n0); t += waves)
    choose(part + t * E16, sigmoid ? part + logits + t * E16 : nullptr, E, top, scale,
           ids + (int64_t)(n0 + t) * top, weights + (int64_t)(n0 + t) * top);
}

// Any dtype: a workgroup per token, a wave per expert in turn.
template <typename T>
__global__ __launch_bounds__(256) void route_plain_kernel(
    int* __restrict__ ids, float* __restrict__ weights, const T* __restrict__ h,
    const T* __restrict__ w, const float* __restrict__ bias, const int E, const int K,
    const int top, const int64_t h_stride, const bool sigmoid, const float scale) {
  extern __shared__ float part[];  // [2][E]
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int64_t n = blockIdx.x;
  for (int e = wid; e < E; e += 4) {
    float z = 0.f;
    for (int k = lane; k < K; k += 64) z += to_f(h[n * h_stride + k]) * to_f(w[(int64_t)e * K + k]);
    z = wave_sum(z);
    if (sigmoid) z = 1.f / (1.f + expf(-z));
    if (lane == 0) {
      part[E + e] = z;
      part[e] = z + (bias ? bias[e] : 0.f);
    }
  }
  __syncthreads();
  if (wid == 0)
    choose(part, sigmoid ? part + E : nullptr, E, top, scale, ids + n * top, weights + n * top);
}

// lanes of the wave whose id (``bits`` bits) equals this lane's
static DEV uint64_t same_id(int id, int bits) {
  uint64_t m = ~0ull;
  for (int b = 0; b < bits; ++b) {
    const uint64_t set = __ballot((id >> b) & 1);
    m &= (id >> b) & 1 ? set : ~set;
  }
  return m;
}

// Group the entries by expert, in their order: a counting sort by one workgroup, each
// wave counting and placing its own run of entries.  Dynamic LDS: [17][E] ints.
__global__ __launch_bounds__(1024) void group_kernel(
    int* __restrict__ perm, int* __restrict__ offsets, int* __restrict__ tile_expert,
    int* __restrict__ tile_row, const int* __restrict__ ids, const int n, const int E) {
  extern __shared__ int counts[];
  int* total = counts + 16 * E;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int bits = 32 - __clz(E);  // E itself marks lanes past the end
  for (int i = threadIdx.x; i < 16 * E; i += 1024) counts[i] = 0;
  __syncthreads();
  const int per = ((n + 15) / 16 + 63) / 64 * 64;
  const int i0 = wid * per, i1 = min(n, i0 + per);
  int* mine = counts + wid * E;
  auto turns = [&](auto&& turn) {  // over this wave's entries, their ids loaded ahead
    for (int i = i0; i < i1; i += 64 * AHEAD) {
      int id[AHEAD];
#pragma unroll
      for (int j = 0; j < AHEAD; ++j) {
        const int at = i + j * 64 + lane;
        id[j] = at < i1 ? ids[at] : E;
      }
#pragma unroll
      for (int j = 0; j < AHEAD; ++j) turn(i + j * 64 + lane, id[j]);
    }
  };
  turns([&](int, int id) {
    const uint64_t m = same_id(id, bits);
    if (id < E && lane == __builtin_ctzll(m)) mine[id] += __popcll(m);
    asm volatile("" ::: "memory");  // the next turn reads what other lanes wrote
  });
  __syncthreads();
  for (int e = threadIdx.x; e < E; e += 1024) {
    int run = 0;
    for (int w = 0; w < 16; ++w) {
      const int t = counts[w * E + e];
      counts[w * E + e] = run;
      run += t;
    }
    total[e] = run;
  }
  __syncthreads();
  if (wid == 0) {  // first rows and tiles of the experts
    int row = 0, tile = 0;
    for (int e0 = 0; e0 < E; e0 += 64) {
      const int e = e0 + lane;
      const int c = e < E ? total[e] : 0, t = (c + EXPERT_TILE - 1) / EXPERT_TILE;
      int cs = c, ts = t;
#pragma unroll
      for (int off = 1; off < 64; off <<= 1) {
        const int a = __shfl_up(cs, off, 64), b = __shfl_up(ts, off, 64);
        if (lane >= off) {
          cs += a;
          ts += b;
        }
      }
      if (e < E) {
        const int first = row + cs - c;
        total[e] = first;
        offsets[e] = first;
        for (int j = 0; j < t && tile_expert; ++j) {
          tile_expert[tile + ts - t + j] = e;
          tile_row[tile + ts - t + j] = first + j * EXPERT_TILE;
        }
      }
      row += __shfl(cs, 63, 64);
      tile += __shfl(ts, 63, 64);
    }
    if (lane == 0) {
      offsets[E] = row;
      offsets[E + 1] = tile;
    }
  }
  __syncthreads();
  turns([&](int at, int id) {
    const uint64_t m = same_id(id, bits);
    const int leader = __builtin_ctzll(m);
    int base = 0;
    if (id < E && lane == leader) {
      base = mine[id];
      mine[id] = base + __popcll(m);
    }
    asm volatile("" ::: "memory");
    base = __shfl(base, leader, 64);
    if (id < E) perm[total[id] + base + __popcll(m & ((1ull << lane) - 1))] = at;
  });
}

// Few rows per expert: bound by the weights.  grid (outputs / 16 or 32, E); the 4 waves
// of a workgroup split K in blocks of 64 and meet in LDS.  Two 16-row weight fragments:
// gate and up of the same 16 outputs, or 32 outputs.  TT token fragments of 16 at a time.
template <bool GLU, int TT>
__global__ __launch_bounds__(256) void experts_small_kernel(const ExpertsArgs a) {
  __shared__ f32x4_v red[4][2][TT][64];
  const int e = blockIdx.y;
  const int row0 = a.offsets[e], rows = a.offsets[e + 1] - row0;
  if (rows == 0) return;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int c = lane & 15, g = lane >> 4;
  const int o0 = blockIdx.x * (GLU ? 16 : 32);
  const bf16_t* w = (const bf16_t*)a.w + (int64_t)e * (GLU ? 2 : 1) * a.O * a.K + g * 8;
  const bf16_t* w0 = w + (int64_t)min(o0 + c, a.O - 1) * a.K;
  const bf16_t* w1 = w + (int64_t)(GLU ? a.O + o0 + c : min(o0 + 16 + c, a.O - 1)) * a.K;
  for (int r0 = 0; r0 < rows; r0 += 16 * TT) {
    const bf16_t* xp[TT];
#pragma unroll
    for (int t = 0; t < TT; ++t) {
      const int r = row0 + min(r0 + t * 16 + c, rows - 1);
      xp[t] = (const bf16_t*)a.x + (int64_t)(GLU ? a.perm[r] / a.top : r) * a.x_stride + g * 8;
    }
    f32x4_v acc[2][TT] = {};
#pragma unroll 2
    for (int k = wid * 64; k < a.K; k += 256) {
#pragma unroll
      for (int s = 0; s < 64; s += 32) {
        const bf16x8_v f0 = *(const bf16x8_v*)(w0 + k + s);
        const bf16x8_v f1 = *(const bf16x8_v*)(w1 + k + s);
#pragma unroll
        for (int t = 0; t < TT; ++t) {
          const bf16x8_v b = *(const bf16x8_v*)(xp[t] + k + s);
          acc[0][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f0, b, acc[0][t], 0, 0, 0);
          acc[1][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f1, b, acc[1][t], 0, 0, 0);
        }
      }
    }
    if (r0) __syncthreads();
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int t = 0; t < TT; ++t) red[wid][i][t][lane] = acc[i][t];
    __syncthreads();
    // a thread sums 4 outputs of one row
    for (int j = threadIdx.x; j < (GLU ? 1 : 2) * TT * 64; j += 256) {
      const int l = j & 63, t = (j >> 6) % TT, i = (j >> 6) / TT;
      const int r = r0 + t * 16 + (l & 15), o = o0 + i * 16 + (l >> 4) * 4;
      if (r >= rows || o >= a.O) continue;
      f32x4_v v = red[0][i][t][l] + red[1][i][t][l] + red[2][i][t][l] + red[3][i][t][l];
      float y[4] = {v[0], v[1], v[2], v[3]};
      if (GLU) {
        v = red[0][1][t][l] + red[1][1][t][l] + red[2][1][t][l] + red[3][1][t][l];
#pragma unroll
        for (int k = 0; k < 4; ++k) {  // through the model's precision, as a GEMM stores it
          const float gate = to_f(from_f<bf16_t>(y[k])), up = to_f(from_f<bf16_t>(v[k]));
          y[k] = clamped_glu_f(gate, up, a.limit, a.alpha, a.offset, a.cubic);
        }
      }
      const int64_t row = GLU ? row0 + r : a.perm[row0 + r];
      bf16_t* dst = (bf16_t*)a.out + row * a.O + o;
      if (a.O % 4 == 0)
        store_f<4>(dst, y);
      else
        for (int k = 0; k < 4 && o + k < a.O; ++k) dst[k] = from_f<bf16_t>(y[k]);
    }
  }
}

// fp32: a thread per output; rows are entries in both products, nothing is grouped.
template <bool GLU>
__global__ __launch_bounds__(256) void experts_f32_kernel(const ExpertsArgs a) {
  const int o = blockIdx.y * 64 + (threadIdx.x & 63);
  const int i = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (o >= a.O || i >= a.entries) return;
  const float* w = (const float*)a.w + ((int64_t)a.ids[i] * (GLU ? 2 : 1) * a.O + o) * a.K;
  const float* x = (const float*)a.x + (int64_t)(GLU ? i / a.top : i) * a.x_stride;
  float g = 0.f, u = 0.f;
  for (int k = 0; k < a.K; k += 4) {
    float xv[4], wv[4];
    load_f<4>(xv, x + k);
    load_f<4>(wv, w + k);
#pragma unroll
    for (int j = 0; j < 4; ++j) g += xv[j] * wv[j];
    if (GLU) {
      load_f<4>(wv, w + (int64_t)a.O * a.K + k);
#pragma unroll
      for (int j = 0; j < 4; ++j) u += xv[j] * wv[j];
    }
  }
  ((float*)a.out)[(int64_t)i * a.O + o] =
      GLU ? clamped_glu_f(g, u, a.limit, a.alpha, a.offset, a.cubic) : g;
}

extern "C" {

void launch_moe_route(bool bf16, int* ids, float* weights, const void* h, const void* w,
                      const float* bias, int N, int E, int K, int top, int64_t h_stride,
                      bool sigmoid, float scale, hipStream_t stream) {
  const int E16 = (E + 15) & ~15;
  if (bf16 && E <= 128) {  // at most 64 KiB of partial logits
    // few workgroups: more waves share the weights' latency
    const int waves = N <= 4096 && E16 <= 64 ? 16 : 8;
    auto k = E16 <= 16   ? route_mfma_kernel<1>
             : E16 <= 32 ? route_mfma_kernel<2>
                         : route_mfma_kernel<4>;
    k<<<(N + ROUTE_T - 1) / ROUTE_T, 64 * waves, waves * ROUTE_T * E16 * 4, stream>>>(
        ids, weights, (const bf16_t*)h, (const bf16_t*)w, bias, N, E, K, top, h_stride, sigmoid,
        scale);
  } else if (bf16) {
    route_plain_kernel<bf16_t><<<N, 256, E * 8, stream>>>(
        ids, weights, (const bf16_t*)h, (const bf16_t*)w, bias, E, K, top, h_stride, sigmoid,
        scale);
  } else {
    route_plain_kernel<float><<<N, 256, E * 8, stream>>>(
        ids, weights, (const float*)h, (const float*)w, bias, E, K, top, h_stride, sigmoid,
        scale);
  }
}

void launch_moe_group(int* perm, int* offsets, int* tile_expert, int* tile_row, const int* ids,
                      int n, int E, hipStream_t stream) {
  group_kernel<<<1, 1024, 17 * E * 4, stream>>>(perm, offsets, tile_expert, tile_row, ids, n, E);
}

// tt: token fragments at a time, 1 or 2
void launch_experts_small(bool glu, const ExpertsArgs* a, int tt, hipStream_t stream) {
  const int per = glu ? 16 : 32;
  const dim3 grid((a->O + per - 1) / per, a->E);
  auto k = glu ? (tt == 1 ? experts_small_kernel<true, 1> : experts_small_kernel<true, 2>)
               : (tt == 1 ? experts_small_kernel<false, 1> : experts_small_kernel<false, 2>);
  k<<<grid, 256, 0, stream>>>(*a);
}

void launch_experts_f32(bool glu, const ExpertsArgs* a, hipStream_t stream) {
  const dim3 grid((a->entries + 3) / 4, (a->O + 63) / 64);
  auto k = glu ? experts_f32_kernel<true> : experts_f32_kernel<false>;
  k<<<grid, 256, 0, stream>>>(*a);
}

}  // extern "C"
