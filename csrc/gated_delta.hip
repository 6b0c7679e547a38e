// Gated delta rule with a decay per head and key channel, or one per head (gfx950).
//
//   S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//
// per head, S [D, V] in fp32.  With k and q known ahead, both products of a token are
// taken over the decayed state at once: o = (diag(g) S)^T q + (k . q) u, so a token
// costs one reduction.  One decay per head is a factor on both sums and needs no vector
// of its own.  Everything in the recurrence is fp32 (the VALU's rate, since
// the bf16 matrix cores would round q, k and S).
//
// Portions of a prompt, three launches:
//   delta_inputs: short convolution + silu, unit factors, k . q, decays per channel
//   delta_scan:   the recurrence.  A wave owns 4 * CPL columns of S in registers, 16
//                 lanes a column; q, k, g of the head's next tokens wait in LDS, shared
//                 by the workgroup's columns
//   delta_output: norm over the head and gate
// One token per sequence: delta_step does all of it, S once through registers.
//
// The convolution's inputs are kept in a ring by position, so that a token's write
// never hits an entry that the token's own convolution reads, whichever workgroup
// comes first.
#include "common_t.h"
#include "gated_delta.h"

DEV float silu_f(float x) { return x * __builtin_amdgcn_rcpf(1.f + __expf(-x)); }

// log(1 + e^x) with a small relative error everywhere: log(u) e / (u - 1), u = 1 + e
DEV float softplus_f(float x) {
  if (x > 20.f) return x;
  const float e = __expf(x), u = 1.f + e;
  return u == 1.f ? e : __logf(u) * e * __builtin_amdgcn_rcpf(u - 1.f);
}

DEV float gate_f(float x, bool silu) { return (silu ? x : 1.f) * sigmoid_f(x); }

// rate = exp(A_log)
DEV float decay_f(float z, float rate) { return __expf(-rate * softplus_f(z)); }

// Where a token's convolution finds its inputs: ``back`` rows before ``row`` belong to
// this step, older ones are in the ring.  p: the token's position.
template <typename T>
struct ConvInput {
  const T* row;
  const T* ring;
  int p, back, taps, C;
  int64_t stride;
  // input ``ago`` tokens earlier, or null before the start
  DEV const T* at(int ago) const {
    if (ago <= back) return row - ago * stride;
    return ago > p ? nullptr : ring + (int64_t)((p - ago) % taps) * C;
  }
};

// convolution of channels c .. c + VW - 1, rounded as the model stores it; TAPS = 0:
// any number
template <typename T, int VW, int TAPS>
DEV void conv_silu(float* y, const T* conv, const ConvInput<T>& in, int c) {
#pragma unroll
  for (int k = 0; k < VW; ++k) y[k] = 0.f;
  if constexpr (TAPS > 0) {
    // all loads first
    Pack<T, VW> x[TAPS];
    Pack<T, TAPS> w[VW];
    bool have[TAPS];
#pragma unroll
    for (int n = 0; n < TAPS; ++n) {
      const T* src = in.at(TAPS - 1 - n);
      have[n] = src;
      x[n] = *(const Pack<T, VW>*)((src ? src : in.row) + c);
    }
#pragma unroll
    for (int k = 0; k < VW; ++k) w[k] = *(const Pack<T, TAPS>*)(conv + (int64_t)(c + k) * TAPS);
#pragma unroll
    for (int n = 0; n < TAPS; ++n)
#pragma unroll
      for (int k = 0; k < VW; ++k) y[k] += have[n] ? to_f(w[k].v[n]) * to_f(x[n].v[k]) : 0.f;
  } else {
    for (int n = 0; n < in.taps; ++n) {
      const T* src = in.at(in.taps - 1 - n);
      if (!src) continue;
      float x[VW];
      load_f<VW>(x, src + c);
#pragma unroll
      for (int k = 0; k < VW; ++k) y[k] += to_f(conv[(int64_t)(c + k) * in.taps + n]) * x[k];
    }
  }
#pragma unroll
  for (int k = 0; k < VW; ++k) y[k] = to_f(from_f<T>(silu_f(y[k])));
}

// ---------------------------------------------------------------- prompts

// grid (tiles of 16 tokens, G + 2 H): a wave per token and head.  The first G heads
// are q and k together, the next H v, the last H the decays per channel.
template <typename T, int VW>
__global__ __launch_bounds__(256) void delta_inputs_kernel(const DeltaArgs a) {
  const int tile = blockIdx.x, job = blockIdx.y;
  const int seq = a.tile_seq[tile], q0 = a.tile_q0[tile];
  const int ctx = a.ctx_lens[seq], len = a.seq_lens[seq] - ctx;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const T* ring = (const T*)a.ring + (int64_t)a.slots[seq] * a.taps * a.C;
  const T* conv = (const T*)a.conv;
  for (int i = wid; i < 16; i += 4) {
    const int t = q0 + i;
    if (t >= len) return;
    const int64_t n = a.row_starts[seq] + t;
    if (job >= a.G + a.H) {
      const int h = job - a.G - a.H;
      const float rate = expf(a.A_log[h]);
      const T* z = (const T*)a.z + n * a.z_stride + (int64_t)h * a.D;
      float* g = a.g + (n * a.H + h) * a.D;
      for (int d = lane * VW; d < a.D; d += 64 * VW) {
        float v[VW];
        load_f<VW>(v, z + d);
#pragma unroll
        for (int k = 0; k < VW; ++k) v[k] = decay_f(v[k] + a.dt_bias[h * a.D + d + k], rate);
        store_f<VW>(g + d, v);
      }
      continue;
    }
    const ConvInput<T> in = {(const T*)a.qkv + n * a.qkv_stride, ring, ctx + t, t, a.taps, a.C,
                             a.qkv_stride};
    T* y = (T*)a.y + n * a.C;
    if (job >= a.G) {
      const int c0 = 2 * a.G * a.D + (job - a.G) * a.V;
      for (int d = lane * VW; d < a.V; d += 64 * VW) {
        float v[VW];
        conv_silu<T, VW, 0>(v, conv, in, c0 + d);
        store_f<VW>(y + c0 + d, v);
      }
      continue;
    }
    const int cq = job * a.D, ck = (a.G + job) * a.D;
    float qq = 0.f, kk = 0.f, kq = 0.f;
    for (int d = lane * VW; d < a.D; d += 64 * VW) {
      float q[VW], k[VW];
      conv_silu<T, VW, 0>(q, conv, in, cq + d);
      conv_silu<T, VW, 0>(k, conv, in, ck + d);
      store_f<VW>(y + cq + d, q);
      store_f<VW>(y + ck + d, k);
#pragma unroll
      for (int e = 0; e < VW; ++e) {
        qq += q[e] * q[e];
        kk += k[e] * k[e];
        kq += k[e] * q[e];
      }
    }
    const float rq = a.q_scale * rsqrtf(wave_sum(qq) + a.unit_eps);
    const float rk = rsqrtf(wave_sum(kk) + a.unit_eps);
    kq = wave_sum(kq) * rq * rk;
    if (lane < 3) a.unit[(n * a.G + job) * 3 + lane] = lane == 0 ? rq : lane == 1 ? rk : kq;
  }
}

// The same for the usual sizes: 4 taps, heads of at most 16 vectors of VW channels.  A
// thread owns VW channels (16 of them a key head, q and k together) and walks the tile's
// tokens, so that every input is loaded once, a token ahead.
template <typename T, int VW>
__global__ __launch_bounds__(256) void delta_inputs_wide_kernel(const DeltaArgs a) {
  const int tile = blockIdx.x;
  const int seq = a.tile_seq[tile], q0 = a.tile_q0[tile];
  const int ctx = a.ctx_lens[seq], n = min(16, a.seq_lens[seq] - ctx - q0);
  const int64_t row0 = a.row_starts[seq] + q0;
  int unit = blockIdx.y * 256 + threadIdx.x;

  if (unit >= a.G * 16 + a.H * a.V / VW) {  // decays per channel
    if (a.head_decay) return;
    const int c = (unit - a.G * 16 - a.H * a.V / VW) * VW;
    if (c >= a.H * a.D) return;
    const float rate = expf(a.A_log[c / a.D]);
    float bias[VW];
#pragma unroll
    for (int k = 0; k < VW; ++k) bias[k] = a.dt_bias[c + k];
    const T* z = (const T*)a.z + row0 * a.z_stride + c;
    float* g = a.g + row0 * a.H * a.D + c;
    Pack<T, VW> next = *(const Pack<T, VW>*)z;
    for (int t = 0; t < n; ++t) {
      const Pack<T, VW> x = next;
      if (t + 1 < n) next = *(const Pack<T, VW>*)(z + (t + 1) * a.z_stride);
      float v[VW];
#pragma unroll
      for (int k = 0; k < VW; ++k) v[k] = decay_f(to_f(x.v[k]) + bias[k], rate);
#pragma unroll
      for (int k = 0; k < VW; k += 4) store_f<4>(g + (int64_t)t * a.H * a.D + k, v + k);
    }
    return;
  }

  const ConvInput<T> in = {(const T*)a.qkv + row0 * a.qkv_stride,
                           (const T*)a.ring + (int64_t)a.slots[seq] * 4 * a.C, ctx + q0, q0, 4,
                           a.C, a.qkv_stride};
  struct Channels {
    float w[4][VW], past[3][VW];
    Pack<T, VW> next;
    int c;
  };
  auto open = [&](Channels& s, int c) {
    s.c = c;
    const T* w = (const T*)a.conv + (int64_t)c * 4;
#pragma unroll
    for (int k = 0; k < VW; ++k) {
      float t[4];
      load_f<4>(t, w + 4 * k);
#pragma unroll
      for (int i = 0; i < 4; ++i) s.w[i][k] = t[i];
    }
#pragma unroll
    for (int i = 0; i < 3; ++i) {
      const T* src = in.at(3 - i);
#pragma unroll
      for (int k = 0; k < VW; ++k) s.past[i][k] = 0.f;
      if (src) load_f<VW>(s.past[i], src + c);
    }
    s.next = *(const Pack<T, VW>*)(in.row + c);
  };
  auto advance = [&](Channels& s, float* y, int t) {
    const Pack<T, VW> x = s.next;
    if (t + 1 < n) s.next = *(const Pack<T, VW>*)(in.row + (t + 1) * a.qkv_stride + s.c);
#pragma unroll
    for (int k = 0; k < VW; ++k) {
      const float v = to_f(x.v[k]);
      y[k] = 0.f;
#pragma unroll
      for (int i = 0; i < 3; ++i) y[k] += s.w[i][k] * s.past[i][k];
      y[k] += s.w[3][k] * v;
      s.past[0][k] = s.past[1][k];
      s.past[1][k] = s.past[2][k];
      s.past[2][k] = v;
      y[k] = to_f(from_f<T>(silu_f(y[k])));
    }
    store_f<VW>((T*)a.y + (row0 + t) * a.C + s.c, y);
  };

  if (unit >= a.G * 16) {  // v
    Channels v;
    open(v, 2 * a.G * a.D + (unit - a.G * 16) * VW);
    float y[VW];
    for (int t = 0; t < n; ++t) advance(v, y, t);
    return;
  }
  const int head = unit >> 4, j = unit & 15;
  const bool live = j * VW < a.D;
  const int d = head * a.D + (live ? j * VW : 0);
  Channels q, k;
  open(q, d);
  open(k, a.G * a.D + d);
  for (int t = 0; t < n; ++t) {
    float yq[VW], yk[VW], qq = 0.f, kk = 0.f, kq = 0.f;
    if (live) {
      advance(q, yq, t);
      advance(k, yk, t);
#pragma unroll
      for (int e = 0; e < VW; ++e) {
        qq += yq[e] * yq[e];
        kk += yk[e] * yk[e];
        kq += yk[e] * yq[e];
      }
    }
    const float rq = a.q_scale * rsqrtf(row16_sum(qq) + a.unit_eps);
    const float rk = rsqrtf(row16_sum(kk) + a.unit_eps);
    kq = row16_sum(kq) * rq * rk;
    if (j < 3)
      a.unit[((row0 + t) * a.G + head) * 3 + j] = j == 0 ? rq : j == 1 ? rk : kq;
  }
}

// N elements as they were loaded, in whole words: taking them apart any earlier than
// needed would wait for the load.
template <typename T, int N>
struct Words {
  static constexpr int COUNT = (N * sizeof(T) + 3) / 4;
  unsigned w[COUNT];
  DEV void load(const T* p) {
    if constexpr (N * sizeof(T) == 2) {
      w[0] = *(const unsigned short*)p;
    } else {
      const Pack<unsigned, COUNT> x = *(const Pack<unsigned, COUNT>*)p;
#pragma unroll
      for (int i = 0; i < COUNT; ++i) w[i] = x.v[i];
    }
  }
  DEV float at(int i) const {
    if (sizeof(T) == 4) return __uint_as_float(w[i]);
    return __uint_as_float(i & 1 ? w[i >> 1] & 0xffff0000u : w[i >> 1] << 16);
  }
};

// grid (column blocks, H, seqs).  Lane j of a column's 16 holds the dims
// (e / VW) * 16 VW + j VW + e % VW: its LDS reads are VW wide and 16 lanes contiguous.
// FULL: D = 16 DPL and rows are aligned to VW channels.  HEAD: one decay per head.
template <typename T, int DPL, int CPL, bool FULL, bool HEAD>
__global__ __launch_bounds__(256) void delta_scan_kernel(const DeltaArgs a) {
  constexpr int TT = DPL <= 16 ? 16 : 256 / DPL;  // tokens staged at a time
  constexpr int DP = 16 * DPL;
  constexpr int VW = DPL < 4 ? DPL : 4, NV = DPL / VW;
  constexpr int COLS = 16 * CPL, SIDE = COLS + 4;
  constexpr int VECS = HEAD ? 2 : 3;
  extern __shared__ float lds[];
  float* const side0 = lds + 2 * VECS * TT * DP;  // per token: v columns, beta, k . q, decay
  const int seq = blockIdx.z, h = blockIdx.y, kvh = h / (a.H / a.G);
  const int ctx = a.ctx_lens[seq], len = a.seq_lens[seq] - ctx;
  const int64_t row0 = a.row_starts[seq], slot = a.slots[seq];
  const int tid = threadIdx.x, j = tid & 15;
  const int col0 = blockIdx.x * COLS, mine = (tid >> 4) * CPL;  // of the workgroup's columns
  auto dim = [&](int e) { return e / VW * (16 * VW) + j * VW + e % VW; };

  float* S = a.state + (slot * a.H + h) * a.D * a.V;
  float s[CPL][DPL];
#pragma unroll
  for (int c = 0; c < CPL; ++c)
#pragma unroll
    for (int e = 0; e < DPL; ++e) {
      const int col = col0 + mine + c;
      s[c][e] = ctx > 0 && dim(e) < a.D && col < a.V ? S[(int64_t)dim(e) * a.V + col] : 0.f;
    }

  // staging: a thread brings its dims and columns of one token (16 threads a token)
  const int tok = tid >> 4;
  constexpr int PW = FULL ? VW : 1, PV = DPL / PW;  // pieces of a thread's dims
  Words<T, PW> rq[PV], rk[PV];
  Words<float, PW> rg[PV];
  Words<T, 1> rv[CPL], fb, fz;
  const float rate = HEAD ? expf(a.A_log[h]) : 0.f, z_bias = HEAD ? a.dt_bias[h] : 0.f;
  float fq, fk, fkq;
  const int t_in = min(tok, len - 1);  // where this thread reads on past the end
  const T* py = (const T*)a.y + (row0 + t_in) * a.C;
  const T* pq = py + kvh * a.D;
  const T* pk = py + (a.G + kvh) * a.D;
  const T* pv = py + 2 * a.G * a.D + h * a.V;
  const float* pg = HEAD ? nullptr : a.g + ((row0 + t_in) * a.H + h) * a.D;
  const T* pz = (const T*)a.z + (row0 + t_in) * a.z_stride + h;
  const float* pu = a.unit + ((row0 + t_in) * a.G + kvh) * 3;
  const T* pb = (const T*)a.b + (row0 + t_in) * a.b_stride + h;
  const int64_t y_step = (int64_t)TT * a.C, g_step = (int64_t)TT * a.H * a.D;
  const int64_t b_step = TT * a.b_stride, z_step = TT * a.z_stride;
  const int u_step = TT * a.G * 3;
  auto fetch = [&](int t0) {
#pragma unroll
    for (int i = 0; i < PV; ++i) {
      const int d = FULL ? dim(i * PW) : min(dim(i * PW), a.D - 1);
      rq[i].load(pq + d);
      rk[i].load(pk + d);
      if (!HEAD) rg[i].load(pg + d);
    }
#pragma unroll
    for (int c = 0; c < CPL; ++c) rv[c].load(pv + min(col0 + j * CPL + c, a.V - 1));
    fq = pu[0];
    fk = pu[1];
    fkq = pu[2];
    fb.load(pb);
    if (HEAD) fz.load(pz);
    if (t0 + TT + tok < len) {
      pq += y_step;
      pk += y_step;
      pv += y_step;
      if (!HEAD) pg += g_step;
      pu += u_step;
      pb += b_step;
      if (HEAD) pz += z_step;
    }
  };
  // tokens past the end change nothing: g = 1, k = q = beta = 0
  auto put = [&](int buf, int t0) {
    if (tok >= TT) return;
    const bool in = t0 + tok < len;
    float* at = lds + (buf * VECS * TT + tok) * DP;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int d = dim(i * VW);
      Pack<float, VW> q, k, g;
#pragma unroll
      for (int e = 0; e < VW; ++e) {
        const int p = (i * VW + e) / PW, o = e % PW;
        const bool has = in && (FULL || d + e < a.D);
        q.v[e] = has ? rq[p].at(o) * fq : 0.f;
        k.v[e] = has ? rk[p].at(o) * fk : 0.f;
        if (!HEAD) g.v[e] = has ? rg[p].at(o) : 1.f;
      }
      *(Pack<float, VW>*)(at + d) = q;
      *(Pack<float, VW>*)(at + TT * DP + d) = k;
      if (!HEAD) *(Pack<float, VW>*)(at + 2 * TT * DP + d) = g;
    }
    float* side = side0 + (buf * TT + tok) * SIDE;
#pragma unroll
    for (int c = 0; c < CPL; ++c) side[j * CPL + c] = rv[c].at(0);
    if (j == 0) {
      side[COLS] = in ? sigmoid_f(fb.at(0)) : 0.f;
      side[COLS + 1] = in ? fkq : 0.f;
      if (HEAD) side[COLS + 2] = in ? decay_f(fz.at(0) + z_bias, rate) : 1.f;
    }
  };

  struct Token {
    float q[DPL], k[DPL], g[HEAD ? 1 : DPL], v[CPL], beta, kq;
  };
  float* po = a.o + ((row0 + j) * a.H + h) * a.V + col0 + mine;  // token j of a chunk
  fetch(0);
  put(0, 0);
  __syncthreads();
  for (int t0 = 0, buf = 0; t0 < len; t0 += TT, buf ^= 1) {
    const bool more = t0 + TT < len;
    if (more) fetch(t0 + TT);
    const int n = min(TT, len - t0);
    float keep[CPL] = {};  // lane j: the output of token j
    auto load = [&](Token& x, int t) {
      const float* at = lds + (buf * VECS * TT + t) * DP + j * VW;
      const float* side = side0 + (buf * TT + t) * SIDE;
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        load_f<VW>(x.q + i * VW, at + i * 16 * VW);
        load_f<VW>(x.k + i * VW, at + TT * DP + i * 16 * VW);
        if constexpr (!HEAD) load_f<VW>(x.g + i * VW, at + 2 * TT * DP + i * 16 * VW);
      }
#pragma unroll
      for (int c = 0; c < CPL; ++c) x.v[c] = side[mine + c];
      x.beta = side[COLS];
      x.kq = side[COLS + 1];
      if (HEAD) x.g[0] = side[COLS + 2];
    };
    auto run = [&](const Token& x, int t) {
#pragma unroll
      for (int c = 0; c < CPL; ++c) {
        float sk = 0.f, sq = 0.f;
#pragma unroll
        for (int e = 0; e < DPL; ++e) {
          if (!HEAD) s[c][e] *= x.g[e];
          sk += x.k[e] * s[c][e];
          sq += x.q[e] * s[c][e];
        }
        sk = row16_sum(sk) * (HEAD ? x.g[0] : 1.f);
        sq = row16_sum(sq) * (HEAD ? x.g[0] : 1.f);
        const float u = x.beta * (x.v[c] - sk);
        const float o = sq + x.kq * u;
        keep[c] = j == t ? o : keep[c];
#pragma unroll
        for (int e = 0; e < DPL; ++e)
          s[c][e] = HEAD ? x.g[0] * s[c][e] + x.k[e] * u : s[c][e] + x.k[e] * u;
      }
    };
    // a token's operands are read while the one before is worked on
    Token even, odd;
    load(even, 0);
    for (int t = 0; t < n; t += 2) {
      load(odd, t + 1);
      __builtin_amdgcn_sched_barrier(0);
      run(even, t);
      load(even, min(t + 2, TT - 1));
      __builtin_amdgcn_sched_barrier(0);
      run(odd, t + 1);
    }
    if (j < n) {
#pragma unroll
      for (int c = 0; c < CPL; ++c)
        if (col0 + mine + c < a.V) po[c] = keep[c];
    }
    po += (int64_t)TT * a.H * a.V;
    if (more) put(buf ^ 1, t0 + TT);
    __syncthreads();
  }

#pragma unroll
  for (int c = 0; c < CPL; ++c)
#pragma unroll
    for (int e = 0; e < DPL; ++e) {
      const int col = col0 + mine + c;
      if (dim(e) < a.D && col < a.V) S[(int64_t)dim(e) * a.V + col] = s[c][e];
    }

  // the head's last convolution inputs; delta_inputs has read the old ones
  if (blockIdx.x == 0) {
    const int group = a.H / a.G;
    const int total = (h % group == 0 ? 2 * a.D : 0) + a.V;
    T* ring = (T*)a.ring + slot * a.taps * a.C;
    for (int i = tid; i < total; i += 256) {
      const int c = i < a.V ? 2 * a.G * a.D + h * a.V + i
                  : i < a.V + a.D ? kvh * a.D + i - a.V : (a.G + kvh) * a.D + i - a.V - a.D;
      for (int t = max(0, len - a.taps); t < len; ++t)
        ring[(int64_t)((ctx + t) % a.taps) * a.C + c] =
            ((const T*)a.qkv)[(row0 + t) * a.qkv_stride + c];
    }
  }
}

// LANES lanes per token and head, 16 or a wave.
template <typename T, int VW, int LANES>
__global__ __launch_bounds__(256) void delta_output_kernel(const DeltaArgs a) {
  const int64_t i = (int64_t)blockIdx.x * (256 / LANES) + threadIdx.x / LANES;
  if (i >= (int64_t)a.N * a.H) return;
  const int64_t n = i / a.H;
  const int h = (int)(i - n * a.H), lane = threadIdx.x % LANES;
  const float* o = a.o + i * a.V;
  const T* gate = (const T*)a.gate + n * a.gate_stride + (int64_t)h * a.V;
  float ss = 0.f;
  for (int d = lane * VW; d < a.V; d += LANES * VW) {
    float x[VW];
    load_f<VW>(x, o + d);
#pragma unroll
    for (int k = 0; k < VW; ++k) ss += x[k] * x[k];
  }
  const float inv = rsqrtf((LANES == 16 ? row16_sum(ss) : wave_sum(ss)) / a.V + a.eps);
  T* out = (T*)a.out + i * a.V;
  for (int d = lane * VW; d < a.V; d += LANES * VW) {
    float x[VW], g[VW], w[VW];
    load_f<VW>(x, o + d);
    load_f<VW>(g, gate + d);
    load_f<VW>(w, a.norm + d);
#pragma unroll
    for (int k = 0; k < VW; ++k) x[k] *= inv * w[k] * gate_f(g[k], a.gate_silu);
    store_f<VW>(out + d, x);
  }
}

// ----------------------------------------------------------------- decode

// grid (H, seqs): a thread owns VW columns of every RG-th row of S, at most ROWS rows;
// ROWS = 0: any number, S is read twice.
template <typename T, int VW, int ROWS, int TAPS>
__global__ __launch_bounds__(1024) void delta_step_kernel(const DeltaArgs a) {
  extern __shared__ float lds[];
  const int h = blockIdx.x, seq = blockIdx.y;
  const int group = a.H / a.G, kvh = h / group;
  const int tid = threadIdx.x, threads = blockDim.x;
  const int lane = tid & 63, wid = tid >> 6, waves = threads >> 6;
  const int ct = a.V / VW, RG = threads / ct;
  const int rg = tid / ct, col = (tid - rg * ct) * VW;
  const bool active = rg < RG;
  float* const q = lds;               // [D], unit after the reduction
  float* const k = q + a.D;           // [D]
  float* const g = k + a.D;           // [D]
  float* const v = g + a.D;           // [V], then u
  float* const o = v + a.V;           // [V]
  float* const red = o + a.V;         // [2][RG][V]
  float* const sums = red + 2 * RG * a.V;  // [waves][4]

  const int64_t slot = a.slots[seq];
  float* S = a.state + (slot * a.H + h) * a.D * a.V;
  Pack<float, VW> s[ROWS ? ROWS : 1];
  if (ROWS && active) {
#pragma unroll
    for (int i = 0; i < ROWS; ++i) {
      const int r = rg + i * RG;
      if (r < a.D) s[i] = *(const Pack<float, VW>*)(S + (int64_t)r * a.V + col);
    }
  }

  // convolutions; the input joins the ring
  const int p = a.seq_lens[seq] - 1;
  const T* row = (const T*)a.qkv + seq * a.qkv_stride;
  const T* conv = (const T*)a.conv;
  T* ring = (T*)a.ring + slot * a.taps * a.C;
  T* entry = ring + (int64_t)(p % a.taps) * a.C;
  const ConvInput<T> in = {row, ring, p, 0, a.taps, a.C, 0};
  float qq = 0.f, kk = 0.f, kq = 0.f;
  const float rate = expf(a.A_log[h]);
  for (int d = tid; d < a.D; d += threads) {
    const int cq = kvh * a.D + d, ck = (a.G + kvh) * a.D + d;
    const int hd = a.head_decay ? h : h * a.D + d;
    float y[2];
    conv_silu<T, 1, TAPS>(y, conv, in, cq);
    conv_silu<T, 1, TAPS>(y + 1, conv, in, ck);
    g[d] = decay_f(to_f(((const T*)a.z)[seq * a.z_stride + hd]) + a.dt_bias[hd], rate);
    q[d] = y[0];
    k[d] = y[1];
    if (h == kvh * group) {
      entry[cq] = row[cq];
      entry[ck] = row[ck];
    }
    qq += y[0] * y[0];
    kk += y[1] * y[1];
    kq += y[1] * y[0];
  }
  for (int d = threads - 1 - tid; d < a.V; d += threads) {  // from the other end
    const int c = 2 * a.G * a.D + h * a.V + d;
    float y;
    conv_silu<T, 1, TAPS>(&y, conv, in, c);
    v[d] = y;
    entry[c] = row[c];
  }
  qq = wave_sum(qq);
  kk = wave_sum(kk);
  kq = wave_sum(kq);
  if (lane == 0) {
    sums[wid * 4] = qq;
    sums[wid * 4 + 1] = kk;
    sums[wid * 4 + 2] = kq;
  }
  __syncthreads();
  qq = kk = kq = 0.f;
  for (int w = 0; w < waves; ++w) {
    qq += sums[w * 4];
    kk += sums[w * 4 + 1];
    kq += sums[w * 4 + 2];
  }
  const float fq = a.q_scale * rsqrtf(qq + a.unit_eps), fk = rsqrtf(kk + a.unit_eps);
  kq *= fq * fk;

  // both products over the decayed state
  if (active) {
    float sk[VW] = {}, sq[VW] = {};
    auto add = [&](int r, Pack<float, VW>& x) {
      const float gr = g[r], kr = k[r] * fk, qr = q[r] * fq;
#pragma unroll
      for (int e = 0; e < VW; ++e) {
        x.v[e] *= gr;
        sk[e] += kr * x.v[e];
        sq[e] += qr * x.v[e];
      }
    };
    if (ROWS) {
#pragma unroll
      for (int i = 0; i < ROWS; ++i)
        if (rg + i * RG < a.D) add(rg + i * RG, s[i]);
    } else {
      for (int r = rg; r < a.D; r += RG) {
        s[0] = *(const Pack<float, VW>*)(S + (int64_t)r * a.V + col);
        add(r, s[0]);
      }
    }
#pragma unroll
    for (int e = 0; e < VW; ++e) {
      red[rg * a.V + col + e] = sk[e];
      red[(RG + rg) * a.V + col + e] = sq[e];
    }
  }
  __syncthreads();
  const float beta = sigmoid_f(to_f(((const T*)a.b)[seq * a.b_stride + h]));
  float ss = 0.f;
  for (int d = tid; d < a.V; d += threads) {
    float sk = 0.f, sq = 0.f;
    for (int i = 0; i < RG; ++i) {
      sk += red[i * a.V + d];
      sq += red[(RG + i) * a.V + d];
    }
    const float u = beta * (v[d] - sk);
    v[d] = u;
    o[d] = sq + kq * u;
    ss += o[d] * o[d];
  }
  ss = wave_sum(ss);
  if (lane == 0) sums[wid * 4 + 3] = ss;
  __syncthreads();

  if (active) {
    float u[VW];
#pragma unroll
    for (int e = 0; e < VW; ++e) u[e] = v[col + e];
    auto update = [&](int r, Pack<float, VW>& x) {
      const float kr = k[r] * fk;
#pragma unroll
      for (int e = 0; e < VW; ++e) x.v[e] += kr * u[e];
      *(Pack<float, VW>*)(S + (int64_t)r * a.V + col) = x;
    };
    if (ROWS) {
#pragma unroll
      for (int i = 0; i < ROWS; ++i)
        if (rg + i * RG < a.D) update(rg + i * RG, s[i]);
    } else {
      for (int r = rg; r < a.D; r += RG) {
        s[0] = *(const Pack<float, VW>*)(S + (int64_t)r * a.V + col);
        const float gr = g[r];
#pragma unroll
        for (int e = 0; e < VW; ++e) s[0].v[e] *= gr;
        update(r, s[0]);
      }
    }
  }
  ss = 0.f;
  for (int w = 0; w < waves; ++w) ss += sums[w * 4 + 3];
  const float inv = rsqrtf(ss / a.V + a.eps);
  const T* gate = (const T*)a.gate + seq * a.gate_stride + (int64_t)h * a.V;
  T* out = (T*)a.out + ((int64_t)seq * a.H + h) * a.V;
  for (int d = tid; d < a.V; d += threads)
    out[d] = from_f<T>(o[d] * inv * a.norm[d] * gate_f(to_f(gate[d]), a.gate_silu));
}

// ---------------------------------------------------------------- launches

template <typename T, int DPL, int CPL, bool FULL, bool HEAD>
static void launch_scan(const DeltaArgs& a, hipStream_t stream) {
  constexpr int TT = DPL <= 16 ? 16 : 256 / DPL;
  constexpr int bytes = 4 * (2 * (HEAD ? 2 : 3) * TT * 16 * DPL + 2 * TT * (16 * CPL + 4));
  static_assert(bytes <= 160 * 1024, "LDS");
  static bool attr_set = false;
  if (!attr_set) {
    (void)hipFuncSetAttribute((const void*)delta_scan_kernel<T, DPL, CPL, FULL, HEAD>,
                              hipFuncAttributeMaxDynamicSharedMemorySize, bytes);
    attr_set = true;
  }
  const dim3 grid((a.V + 16 * CPL - 1) / (16 * CPL), a.H, a.seqs);
  delta_scan_kernel<T, DPL, CPL, FULL, HEAD><<<grid, 256, bytes, stream>>>(a);
}

template <typename T, int DPL, bool HEAD>
static void launch_scan_decay(const DeltaArgs& a, int cpl, hipStream_t stream) {
  constexpr int VW = DPL < 4 ? DPL : 4;
  if (a.D != 16 * DPL || a.C % VW != 0)
    launch_scan<T, DPL, 1, false, HEAD>(a, stream);
  else if (cpl == 1 || DPL > 8)
    launch_scan<T, DPL, 1, true, HEAD>(a, stream);
  else if constexpr (DPL <= 8)
    launch_scan<T, DPL, 2, true, HEAD>(a, stream);
}

template <typename T, int DPL>
static void launch_scan_cols(const DeltaArgs& a, int cpl, hipStream_t stream) {
  (a.head_decay ? launch_scan_decay<T, DPL, true> : launch_scan_decay<T, DPL, false>)(a, cpl,
                                                                                      stream);
}

template <typename T>
static void prompts(const DeltaArgs& a, int cpl, hipStream_t stream) {
  constexpr int W = 16 / sizeof(T);
  auto all = [&](int n) {  // every head and row starts at a multiple of n channels
    return a.D % n == 0 && a.V % n == 0 && (a.head_decay || a.z_stride % n == 0) &&
           a.qkv_stride % n == 0 && a.gate_stride % n == 0;
  };
  const uintptr_t z = a.head_decay ? 0 : (uintptr_t)a.z;
  const bool aligned = ((uintptr_t)a.qkv | z | (uintptr_t)a.gate) % 16 == 0;
  if (aligned && all(W) && a.taps == 4 && a.D <= 16 * W) {
    const int units = a.G * 16 + a.H * (a.V + (a.head_decay ? 0 : a.D)) / W;
    delta_inputs_wide_kernel<T, W><<<dim3(a.n_tiles, (units + 255) / 256), 256, 0, stream>>>(a);
  } else {
    const dim3 grid(a.n_tiles, a.G + (a.head_decay ? 1 : 2) * a.H);
    const bool even = all(2) && ((uintptr_t)a.qkv | z) % (2 * sizeof(T)) == 0;
    auto inputs = even ? delta_inputs_kernel<T, 2> : delta_inputs_kernel<T, 1>;
    inputs<<<grid, 256, 0, stream>>>(a);
  }
  if (a.D <= 16) launch_scan_cols<T, 1>(a, cpl, stream);
  else if (a.D <= 32) launch_scan_cols<T, 2>(a, cpl, stream);
  else if (a.D <= 64) launch_scan_cols<T, 4>(a, cpl, stream);
  else if (a.D <= 128) launch_scan_cols<T, 8>(a, cpl, stream);
  else if (a.D <= 256) launch_scan_cols<T, 16>(a, cpl, stream);
  else if (a.D <= 512) launch_scan_cols<T, 32>(a, cpl, stream);
  else launch_scan_cols<T, 64>(a, cpl, stream);
  const int64_t heads = (int64_t)a.N * a.H;
  const bool short_heads = aligned && all(W) && a.V <= 16 * W;
  auto output = short_heads       ? delta_output_kernel<T, W, 16>
                : aligned && all(4) ? delta_output_kernel<T, 4, 64> : delta_output_kernel<T, 1, 64>;
  const int per = short_heads ? 16 : 4;
  output<<<(heads + per - 1) / per, 256, 0, stream>>>(a);
}

template <typename T, int VW, int TAPS>
static void step(const DeltaArgs& a, int threads, hipStream_t stream) {
  const int ct = a.V / VW, RG = threads / ct, rows = (a.D + RG - 1) / RG;
  const int bytes = 4 * (3 * a.D + 2 * a.V + 2 * RG * a.V + threads / 64 * 4);
  const dim3 grid(a.H, a.seqs);
  auto k = rows <= 4    ? delta_step_kernel<T, VW, 4, TAPS>
           : rows <= 8  ? delta_step_kernel<T, VW, 8, TAPS>
           : rows <= 16 ? delta_step_kernel<T, VW, 16, TAPS>
                        : delta_step_kernel<T, VW, 0, TAPS>;
  k<<<grid, threads, bytes, stream>>>(a);
}

template <typename T>
static void step_any(const DeltaArgs& a, int threads, hipStream_t stream) {
  if (a.V % 4 == 0)
    a.taps == 4 ? step<T, 4, 4>(a, threads, stream) : step<T, 4, 0>(a, threads, stream);
  else
    a.taps == 4 ? step<T, 1, 4>(a, threads, stream) : step<T, 1, 0>(a, threads, stream);
}

extern "C" {

// D, V <= 1024
void launch_delta_prompts(bool bf16, const DeltaArgs* a, int cpl, hipStream_t stream) {
  (bf16 ? prompts<bf16_t> : prompts<float>)(*a, cpl, stream);
}

// V % 4 == 0 or V <= threads
void launch_delta_step(bool bf16, const DeltaArgs* a, int threads, hipStream_t stream) {
  (bf16 ? step_any<bf16_t> : step_any<float>)(*a, threads, stream);
}

}  // extern "C"
