// What happens to q, k and v between their projection and attention, in one pass
// (gfx950): short convolution, norms per head or over all heads, rotation, query
// temperature; keys and values go to their cache slots.
//
// A thread owns VW channels of one row.  Heads start at multiples of their size, so a
// head is a group of d / VW neighbouring lanes, which reduce by shuffles; sections are
// aligned so that no group straddles a wave.  Rotations pair dimension 2i with 2i + 1,
// both in one thread.  Norms over all heads take a workgroup per row.  Everything between
// load and store is fp32.
//
// The convolutions' inputs are kept in a ring by position.  A row that is alone in its
// sequence's step writes an entry that its own convolution does not read, at once;
// with longer portions that entry may be one that an earlier row reads, so their last
// inputs follow in a second launch.
#include "common_t.h"
#include "attn_inputs.h"

// input of VW channels ``ago`` > back tokens before row n: from the ring, or zeros
template <typename T, int VW>
DEV Pack<T, VW> ring_input(const AttnInputsArgs& a, int p, int64_t state, int ago, int c) {
  Pack<T, VW> x;
  if (ago <= p) {
    x = *(const Pack<T, VW>*)((const T*)a.ring + (state * a.taps + (p - ago) % a.taps) * a.C + c);
  } else {
#pragma unroll
    for (int k = 0; k < VW; ++k) x.v[k] = from_f<T>(0.f);
  }
  return x;
}

template <typename T, int VW>
DEV Pack<T, VW> row_input(const AttnInputsArgs& a, int64_t n, int c) {
  return *(const Pack<T, VW>*)((const T*)a.proj + n * a.stride + c);
}

template <typename T, int VW>
DEV void add_tap(float* y, const Pack<T, VW>& f, const Pack<T, VW>& x) {
#pragma unroll
  for (int k = 0; k < VW; ++k) y[k] += to_f(f.v[k]) * to_f(x.v[k]);
}

// VW channels of row n, convolved if there is a convolution
template <typename T, int VW>
DEV void channels(const AttnInputsArgs& a, int64_t n, int p, int back, int64_t state, int c,
                  float* y) {
  if (!a.conv) {
    load_f<VW>(y, (const T*)a.proj + n * a.stride + c);
    return;
  }
  const T* w = (const T*)a.conv + c;
#pragma unroll
  for (int k = 0; k < VW; ++k) y[k] = 0.f;
  for (int j = 0; j < a.taps; ++j) {
    const int ago = a.taps - 1 - j;
    add_tap<T, VW>(y, *(const Pack<T, VW>*)(w + (int64_t)j * a.C),
                   ago <= back ? row_input<T, VW>(a, n - ago, c)
                               : ring_input<T, VW>(a, p, state, ago, c));
  }
}

template <typename T, int VW>
DEV void to_ring(const AttnInputsArgs& a, int64_t n, int p, int64_t state, int c) {
  *(Pack<T, VW>*)((T*)a.ring + (state * a.taps + p % a.taps) * a.C + c) = row_input<T, VW>(a, n, c);
}

// y: VW channels from i of a head whose norm's squares sum to ss; sect 0 q, 1 k, 2 v
template <typename T, int VW>
DEV void finish(const AttnInputsArgs& a, int64_t n, int p, int sect, int head, int i, float ss,
                float* y) {
  if (sect < 2 ? a.q_norm != nullptr : a.v_norm) {
    const int heads = !a.row_norm ? 1 : sect == 0 ? a.H : a.G;
    const float inv = rsqrtf(ss / (sect < 2 ? heads * a.dim : a.vdim) + a.eps);
#pragma unroll
    for (int k = 0; k < VW; ++k) y[k] *= inv;
    if (sect < 2) {
      float w[VW];
      const int at = a.row_norm ? head * a.d + i : i;
      load_f<VW>(w, (const T*)(sect == 0 ? a.q_norm : a.k_norm) + at);
#pragma unroll
      for (int k = 0; k < VW; ++k) y[k] *= w[k];
    }
  }
  if (a.cos_sin && sect < 2) {
    const float* ct = a.cos_sin + (int64_t)p * a.pairs;
    const float* st = ct + a.P * a.pairs;
#pragma unroll
    for (int k = 0; k < VW; k += 2) {
      const int at = (i + k) >> 1;
      if (at < a.pairs) {
        const float co = ct[at], si = st[at], u = y[k], v = y[k + 1];
        y[k] = u * co - v * si;
        y[k + 1] = v * co + u * si;
      }
    }
  }
  if (sect == 0) {
    float f = a.head_mult ? a.head_mult[head] : 1.f;
    if (a.q_every > 0.f) f *= 1.f + a.q_coef * logf(floorf((float)(p + 1) / a.q_every) + 1.f);
#pragma unroll
    for (int k = 0; k < VW; ++k) y[k] *= f;
    store_f<VW>((T*)a.q + (n * a.H + head) * a.d + i, y);
  } else if (sect == 1) {
    store_f<VW>((T*)a.k_cache + (a.slots[n] * a.G + head) * a.d + i, y);
  } else {
    store_f<VW>((T*)a.v_cache + (a.slots[n] * a.G + head) * a.v + i, y);
  }
}

// Head sizes of at most 64 threads, a power of two.  grid (threads of a row / 256, rows / R):
// a row has ``units`` threads, a multiple of 64; a thread does R rows in turn.  TAPS: 0 none,
// 4: its rows' inputs are loaded once, -1 any number.
template <typename T, int VW, int TAPS, int R>
__global__ __launch_bounds__(256) void attn_inputs_kernel(const AttnInputsArgs a, const int units) {
  int u = blockIdx.x * 256 + threadIdx.x;
  if (u >= units) return;
  const int64_t n0 = (int64_t)blockIdx.y * R;
  const int lq = a.d / VW, lv = a.v / VW;
  const int k_at = a.H * lq, v_at = ((a.H + a.G) * lq + lv - 1) / lv * lv;
  int sect = 0, c0 = 0, lanes = lq;
  bool live = true;
  if (u >= v_at) {
    sect = 2;
    u -= v_at;
    c0 = (a.H + a.G) * a.d;
    lanes = lv;
    live = u < a.G * lv;
  } else if (u >= k_at) {
    sect = 1;
    u -= k_at;
    c0 = a.H * a.d;
    live = u < a.G * lq;
  }
  if (!live) u = 0;
  const int c = c0 + u * VW, head = u >> (31 - __clz(lanes)), i = (u & (lanes - 1)) * VW;

  constexpr int W = TAPS > 0 ? TAPS : 1;
  Pack<T, VW> x[R + W - 1], f[W];
  if constexpr (TAPS >= 0) {  // row n0 + r and the W - 1 before it are x[r .. r + W - 1]
#pragma unroll
    for (int r = 0; r < R + W - 1; ++r) {
      const int64_t n = n0 - (W - 1) + r;
      x[r] = row_input<T, VW>(a, min(max(n, (int64_t)0), (int64_t)a.N - 1), c);
    }
  }
  if constexpr (TAPS > 0) {
#pragma unroll
    for (int j = 0; j < TAPS; ++j)
      f[j] = *(const Pack<T, VW>*)((const T*)a.conv + (int64_t)j * a.C + c);
  }
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int64_t n = n0 + r;
    if (n >= a.N) return;
    const int p = (int)a.positions[n];
    const int back = TAPS && a.back ? a.back[n] : 0;
    const int64_t state = TAPS ? a.states[n] : 0;
    float y[VW];
    if constexpr (TAPS < 0) {
      channels<T, VW>(a, n, p, back, state, c, y);
    } else if constexpr (TAPS == 0) {
#pragma unroll
      for (int k = 0; k < VW; ++k) y[k] = to_f(x[r].v[k]);
    } else {
#pragma unroll
      for (int k = 0; k < VW; ++k) y[k] = 0.f;
      if (back >= TAPS - 1) {
#pragma unroll
        for (int j = 0; j < TAPS; ++j) add_tap<T, VW>(y, f[j], x[r + j]);
      } else {  // some inputs are from earlier steps
#pragma unroll
        for (int j = 0; j < TAPS; ++j) {
          const int ago = TAPS - 1 - j;
          add_tap<T, VW>(y, f[j], ago <= back ? x[r + j] : ring_input<T, VW>(a, p, state, ago, c));
        }
      }
    }
    if (TAPS && a.write_ring && live) to_ring<T, VW>(a, n, p, state, c);
    float ss = 0.f;
    if (a.q_norm || a.v_norm) {
#pragma unroll
      for (int k = 0; k < VW; ++k) ss += y[k] * y[k];
#pragma unroll
      for (int off = 1; off < 64; off <<= 1) {
        const float t = __shfl_xor(ss, off, 64);
        if (off < lanes) ss += t;
      }
    }
    if (live) finish<T, VW>(a, n, p, sect, head, i, ss, y);
  }
}

// Any head size (a multiple of VW): a wave per row and head.
template <typename T, int VW>
__global__ __launch_bounds__(256) void attn_inputs_any_kernel(const AttnInputsArgs a) {
  const int64_t n = blockIdx.y;
  int head = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (head >= a.H + 2 * a.G) return;
  const int lane = threadIdx.x & 63;
  int sect = 0, c0 = head * a.d, size = a.d;
  if (head >= a.H + a.G) {
    head -= a.H + a.G;
    sect = 2;
    c0 = (a.H + a.G) * a.d + head * a.v;
    size = a.v;
  } else if (head >= a.H) {
    head -= a.H;
    sect = 1;
  }
  const int p = (int)a.positions[n];
  const int back = a.back ? a.back[n] : 0;
  const int64_t state = a.conv ? a.states[n] : 0;
  float ss = 0.f, y[VW];
  for (int i = lane * VW; i < size; i += 64 * VW) {
    channels<T, VW>(a, n, p, back, state, c0 + i, y);
#pragma unroll
    for (int k = 0; k < VW; ++k) ss += y[k] * y[k];
  }
  ss = wave_sum(ss);
  for (int i = lane * VW; i < size; i += 64 * VW) {
    channels<T, VW>(a, n, p, back, state, c0 + i, y);
    if (a.conv && a.write_ring) to_ring<T, VW>(a, n, p, state, c0 + i);
    finish<T, VW>(a, n, p, sect, head, i, ss, y);
  }
}

// Norms over all heads: a workgroup per row, a thread has every blockDim.x-th VW
// channels, at most PER of them.  No convolution, no norm of v.
template <typename T, int VW, int PER>
__global__ __launch_bounds__(1024) void attn_inputs_row_kernel(const AttnInputsArgs a) {
  __shared__ float scratch[2][16];
  const int64_t n = blockIdx.x;
  const int p = (int)a.positions[n];
  const int units = a.C / VW, q_end = a.H * a.d, k_end = q_end + a.G * a.d;
  Pack<T, VW> x[PER];
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    const int u = threadIdx.x + j * blockDim.x;
    x[j] = row_input<T, VW>(a, n, min(u, units - 1) * VW);
  }
  float qq = 0.f, kk = 0.f;
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    const int c = (threadIdx.x + j * blockDim.x) * VW;
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < VW; ++k) ss += to_f(x[j].v[k]) * to_f(x[j].v[k]);
    qq += c < q_end ? ss : 0.f;
    kk += c >= q_end && c < k_end ? ss : 0.f;
  }
  qq = block_sum(qq, scratch[0]);
  kk = block_sum(kk, scratch[1]);
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    int c = (threadIdx.x + j * blockDim.x) * VW;
    if (c >= a.C) return;
    const int sect = c < q_end ? 0 : c < k_end ? 1 : 2;
    c -= sect == 0 ? 0 : sect == 1 ? q_end : k_end;
    const int size = sect < 2 ? a.d : a.v, head = c / size;
    float y[VW];
#pragma unroll
    for (int k = 0; k < VW; ++k) y[k] = to_f(x[j].v[k]);
    finish<T, VW>(a, n, p, sect, head, c - head * size, sect == 0 ? qq : kk, y);
  }
}

// grid (parts of a row, ring rows)
template <typename T, int VW>
__global__ __launch_bounds__(256) void attn_ring_kernel(const AttnInputsArgs a) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * VW;
  if (c >= a.C) return;
  const int64_t n = a.ring_rows[blockIdx.y];
  to_ring<T, VW>(a, n, (int)a.positions[n], a.states[n], c);
}

template <typename T, int VW, int R>
static void launch_rows(const AttnInputsArgs& a, int units, hipStream_t stream) {
  auto k = !a.conv       ? attn_inputs_kernel<T, VW, 0, R>
           : a.taps == 4 ? attn_inputs_kernel<T, VW, 4, R>
                         : attn_inputs_kernel<T, VW, -1, R>;
  k<<<dim3((units + 255) / 256, (a.N + R - 1) / R), 256, 0, stream>>>(a, units);
}

template <typename T, int VW>
static void launch(const AttnInputsArgs& a, hipStream_t stream) {
  const int lq = a.d / VW, lv = a.v / VW;
  auto fits = [](int lanes) { return lanes <= 64 && (lanes & (lanes - 1)) == 0; };
  if (a.row_norm) {
    const int units = a.C / VW;
    int threads = 256;
    while (threads < 1024 && units > 4 * threads) threads *= 2;
    if (units <= threads)
      attn_inputs_row_kernel<T, VW, 1><<<a.N, threads, 0, stream>>>(a);
    else if (units <= 4 * threads)
      attn_inputs_row_kernel<T, VW, 4><<<a.N, threads, 0, stream>>>(a);
    else
      attn_inputs_row_kernel<T, VW, 16><<<a.N, threads, 0, stream>>>(a);
    return;
  }
  if (fits(lq) && fits(lv)) {
    const int v_at = ((a.H + a.G) * lq + lv - 1) / lv * lv;
    const int units = (v_at + a.G * lv + 63) / 64 * 64;
    if (a.N >= 2048)
      launch_rows<T, VW, 4>(a, units, stream);
    else
      launch_rows<T, VW, 1>(a, units, stream);
  } else {
    attn_inputs_any_kernel<T, VW><<<dim3((a.H + 2 * a.G + 3) / 4, a.N), 256, 0, stream>>>(a);
  }
  if (a.n_ring_rows)
    attn_ring_kernel<T, VW><<<dim3((a.C / VW + 255) / 256, a.n_ring_rows), 256, 0, stream>>>(a);
}

extern "C" void launch_attn_inputs(bool bf16, const AttnInputsArgs* a, hipStream_t stream) {
  bf16 ? launch<bf16_t, 8>(*a, stream) : launch<float, 4>(*a, stream);
}
