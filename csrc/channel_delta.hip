// Gated delta rule with a decay per head and key channel (gfx950).
//
//   S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//
// per head, S [D, V] in fp32.  With k and q known ahead, both products of a token are
// taken over the decayed state at once: o = (diag(g) S)^T q + (k . q) u, so a token
// costs one reduction.  Everything in the recurrence is fp32 (the VALU's rate, since
// the bf16 matrix cores would round q, k and S).
//
// Portions of a prompt, three launches:
//   delta_inputs: short convolution + silu, unit factors, k . q, decays
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
#include "channel_delta.h"

DEV float silu_f(float x) { return x / (1.f + expf(-x)); }
DEV float softplus_f(float x) { return x > 20.f ? x : log1pf(expf(x)); }
DEV float decay_f(float z, float A_log) { return expf(-expf(A_log) * softplus_f(z)); }

// convolution of channels c .. c + VW - 1 at position p, rounded as the model stores it;
// row: the token's input row, ``back`` rows before it are this step's
template <typename T, int VW>
DEV void conv_silu(float* y, const DeltaArgs& a, const T* row, const T* ring, int c, int p,
                   int back) {
  const T* w = (const T*)a.conv + (int64_t)c * a.taps;
#pragma unroll
  for (int k = 0; k < VW; ++k) y[k] = 0.f;
  for (int n = 0; n < a.taps; ++n) {
    const int ago = a.taps - 1 - n;  // tokens before this one
    if (ago > p) continue;
    const T* src = ago <= back ? row - ago * a.qkv_stride
                               : ring + (int64_t)((p - ago) % a.taps) * a.C;
    float x[VW];
    load_f<VW>(x, src + c);
#pragma unroll
    for (int k = 0; k < VW; ++k) y[k] += to_f(w[k * a.taps + n]) * x[k];
  }
#pragma unroll
  for (int k = 0; k < VW; ++k) y[k] = to_f(from_f<T>(silu_f(y[k])));
}

// ---------------------------------------------------------------- prompts

// grid (tiles of 16 tokens, G + 2 H): a wave per token and head.  The first G heads
// are q and k together, the next H v, the last H the decays.
template <typename T, int VW>
__global__ __launch_bounds__(256) void delta_inputs_kernel(const DeltaArgs a) {
  const int tile = blockIdx.x, job = blockIdx.y;
  const int seq = a.tile_seq[tile], q0 = a.tile_q0[tile];
  const int ctx = a.ctx_lens[seq], len = a.seq_lens[seq] - ctx;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const T* ring = (const T*)a.ring + (int64_t)a.slots[seq] * a.taps * a.C;
  for (int i = wid; i < 16; i += 4) {
    const int t = q0 + i;
    if (t >= len) return;
    const int64_t n = a.row_starts[seq] + t;
    if (job >= a.G + a.H) {
      const int h = job - a.G - a.H;
      const float A_log = a.A_log[h];
      const T* z = (const T*)a.z + n * a.z_stride + (int64_t)h * a.D;
      float* g = a.g + (n * a.H + h) * a.D;
      for (int d = lane * VW; d < a.D; d += 64 * VW) {
        float v[VW];
        load_f<VW>(v, z + d);
#pragma unroll
        for (int k = 0; k < VW; ++k) v[k] = decay_f(v[k] + a.dt_bias[h * a.D + d + k], A_log);
        store_f<VW>(g + d, v);
      }
      continue;
    }
    const T* row = (const T*)a.qkv + n * a.qkv_stride;
    T* y = (T*)a.y + n * a.C;
    const int p = ctx + t;
    if (job >= a.G) {
      const int c0 = 2 * a.G * a.D + (job - a.G) * a.V;
      for (int d = lane * VW; d < a.V; d += 64 * VW) {
        float v[VW];
        conv_silu<T, VW>(v, a, row, ring, c0 + d, p, t);
        store_f<VW>(y + c0 + d, v);
      }
      continue;
    }
    const int cq = job * a.D, ck = (a.G + job) * a.D;
    float qq = 0.f, kk = 0.f, kq = 0.f;
    for (int d = lane * VW; d < a.D; d += 64 * VW) {
      float q[VW], k[VW];
      conv_silu<T, VW>(q, a, row, ring, cq + d, p, t);
      conv_silu<T, VW>(k, a, row, ring, ck + d, p, t);
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

// grid (column blocks, H, seqs).  Lane j of a column's 16 holds the dims
// (e / VW) * 16 VW + j VW + e % VW: its LDS reads are VW wide and 16 lanes contiguous.
template <typename T, int DPL, int CPL>
__global__ __launch_bounds__(256) void delta_scan_kernel(const DeltaArgs a) {
  constexpr int TT = DPL <= 16 ? 16 : 256 / DPL;  // tokens staged at a time
  constexpr int DP = 16 * DPL;
  constexpr int VW = DPL < 4 ? DPL : 4, NV = DPL / VW;
  constexpr int COLS = 16 * CPL, SIDE = COLS + 4;
  extern __shared__ float lds[];
  float* const side0 = lds + 2 * 3 * TT * DP;  // per token: v columns, beta, k . q
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
  const bool wide = a.D % VW == 0 && a.C % VW == 0;
  Pack<T, VW> rq[NV], rk[NV];
  Pack<float, VW> rg[NV];
  float rv[CPL], fq, fk, fb, fkq;
  auto fetch = [&](int t0) {
    const int t = t0 + tok;
    const bool in = tok < TT && t < len;
    const int64_t n = row0 + (in ? t : 0);
    const T* y = (const T*)a.y + n * a.C;
    const T* yq = y + kvh * a.D;
    const T* yk = y + (a.G + kvh) * a.D;
    const float* g = a.g + (n * a.H + h) * a.D;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int d = dim(i * VW);
      if (wide) {
        if (d < a.D) {
          rq[i] = *(const Pack<T, VW>*)(yq + d);
          rk[i] = *(const Pack<T, VW>*)(yk + d);
          rg[i] = *(const Pack<float, VW>*)(g + d);
        }
      } else {
#pragma unroll
        for (int k = 0; k < VW; ++k)
          if (d + k < a.D) {
            rq[i].v[k] = yq[d + k];
            rk[i].v[k] = yk[d + k];
            rg[i].v[k] = g[d + k];
          }
      }
    }
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
      const int col = min(col0 + j * CPL + c, a.V - 1);
      rv[c] = to_f(y[2 * a.G * a.D + h * a.V + col]);
    }
    const float* u = a.unit + (n * a.G + kvh) * 3;
    fq = u[0];
    fk = u[1];
    fkq = u[2];
    fb = to_f(((const T*)a.b)[n * a.b_stride + h]);
  };
  auto put = [&](int buf) {
    if (tok >= TT) return;
    float* at = lds + (buf * 3 * TT + tok) * DP;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int d = dim(i * VW);
      Pack<float, VW> q, k, g;
#pragma unroll
      for (int e = 0; e < VW; ++e) {
        const bool in = d + e < a.D;
        q.v[e] = in ? to_f(rq[i].v[e]) * fq : 0.f;
        k.v[e] = in ? to_f(rk[i].v[e]) * fk : 0.f;
        g.v[e] = in ? rg[i].v[e] : 0.f;
      }
      *(Pack<float, VW>*)(at + d) = q;
      *(Pack<float, VW>*)(at + TT * DP + d) = k;
      *(Pack<float, VW>*)(at + 2 * TT * DP + d) = g;
    }
    float* side = side0 + (buf * TT + tok) * SIDE;
#pragma unroll
    for (int c = 0; c < CPL; ++c) side[j * CPL + c] = rv[c];
    if (j == 0) {
      side[COLS] = sigmoid_f(fb);
      side[COLS + 1] = fkq;
    }
  };

  fetch(0);
  put(0);
  __syncthreads();
  for (int t0 = 0, buf = 0; t0 < len; t0 += TT, buf ^= 1) {
    const bool more = t0 + TT < len;
    if (more) fetch(t0 + TT);
    const int n = min(TT, len - t0);
    float keep[CPL] = {};  // lane j: the output of token j
    for (int t = 0; t < n; ++t) {
      const float* at = lds + (buf * 3 * TT + t) * DP + j * VW;
      const float* side = side0 + (buf * TT + t) * SIDE;
      float q[DPL], k[DPL], g[DPL];
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        load_f<VW>(q + i * VW, at + i * 16 * VW);
        load_f<VW>(k + i * VW, at + TT * DP + i * 16 * VW);
        load_f<VW>(g + i * VW, at + 2 * TT * DP + i * 16 * VW);
      }
      const float beta = side[COLS], kq = side[COLS + 1];
#pragma unroll
      for (int c = 0; c < CPL; ++c) {
        float sk = 0.f, sq = 0.f;
#pragma unroll
        for (int e = 0; e < DPL; ++e) {
          s[c][e] *= g[e];
          sk += k[e] * s[c][e];
          sq += q[e] * s[c][e];
        }
        sk = row16_sum(sk);
        sq = row16_sum(sq);
        const float u = beta * (side[mine + c] - sk);
        const float o = sq + kq * u;
        keep[c] = j == t ? o : keep[c];
#pragma unroll
        for (int e = 0; e < DPL; ++e) s[c][e] += k[e] * u;
      }
    }
    if (j < n) {
      float* o = a.o + ((row0 + t0 + j) * a.H + h) * a.V + col0 + mine;
#pragma unroll
      for (int c = 0; c < CPL; ++c)
        if (col0 + mine + c < a.V) o[c] = keep[c];
    }
    if (more) put(buf ^ 1);
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

// A wave per token and head.
template <typename T>
__global__ __launch_bounds__(256) void delta_output_kernel(const DeltaArgs a) {
  const int64_t i = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (i >= (int64_t)a.N * a.H) return;
  const int64_t n = i / a.H;
  const int h = (int)(i - n * a.H), lane = threadIdx.x & 63;
  const float* o = a.o + i * a.V;
  float ss = 0.f;
  for (int d = lane; d < a.V; d += 64) ss += o[d] * o[d];
  const float inv = rsqrtf(wave_sum(ss) / a.V + a.eps);
  const T* gate = (const T*)a.gate + n * a.gate_stride + (int64_t)h * a.V;
  T* out = (T*)a.out + i * a.V;
  for (int d = lane; d < a.V; d += 64)
    out[d] = from_f<T>(o[d] * inv * a.norm[d] * sigmoid_f(to_f(gate[d])));
}

// ----------------------------------------------------------------- decode

// grid (H, seqs): a thread owns VW columns of every RG-th row of S, at most ROWS rows;
// ROWS = 0: any number, S is read twice.
template <typename T, int VW, int ROWS>
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
  T* ring = (T*)a.ring + slot * a.taps * a.C;
  float qq = 0.f, kk = 0.f, kq = 0.f;
  for (int d = tid; d < a.D; d += threads) {
    const int cq = kvh * a.D + d, ck = (a.G + kvh) * a.D + d;
    conv_silu<T, 1>(q + d, a, row, ring, cq, p, 0);
    conv_silu<T, 1>(k + d, a, row, ring, ck, p, 0);
    if (h == kvh * group) {
      ring[(int64_t)(p % a.taps) * a.C + cq] = row[cq];
      ring[(int64_t)(p % a.taps) * a.C + ck] = row[ck];
    }
    qq += q[d] * q[d];
    kk += k[d] * k[d];
    kq += k[d] * q[d];
    const int hd = h * a.D + d;
    g[d] = decay_f(to_f(((const T*)a.z)[seq * a.z_stride + hd]) + a.dt_bias[hd], a.A_log[h]);
  }
  for (int d = tid; d < a.V; d += threads) {
    const int c = 2 * a.G * a.D + h * a.V + d;
    conv_silu<T, 1>(v + d, a, row, ring, c, p, 0);
    ring[(int64_t)(p % a.taps) * a.C + c] = row[c];
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
    out[d] = from_f<T>(o[d] * inv * a.norm[d] * sigmoid_f(to_f(gate[d])));
}

// ---------------------------------------------------------------- launches

template <typename T, int DPL, int CPL>
static void launch_scan(const DeltaArgs& a, hipStream_t stream) {
  constexpr int TT = DPL <= 16 ? 16 : 256 / DPL;
  constexpr int bytes = 4 * (2 * 3 * TT * 16 * DPL + 2 * TT * (16 * CPL + 4));
  static_assert(bytes <= 160 * 1024, "LDS");
  static bool attr_set = false;
  if (!attr_set) {
    (void)hipFuncSetAttribute((const void*)delta_scan_kernel<T, DPL, CPL>,
                              hipFuncAttributeMaxDynamicSharedMemorySize, bytes);
    attr_set = true;
  }
  const dim3 grid((a.V + 16 * CPL - 1) / (16 * CPL), a.H, a.seqs);
  delta_scan_kernel<T, DPL, CPL><<<grid, 256, bytes, stream>>>(a);
}

template <typename T, int DPL>
static void launch_scan_cols(const DeltaArgs& a, int cpl, hipStream_t stream) {
  if (cpl == 1 || DPL > 8)
    launch_scan<T, DPL, 1>(a, stream);
  else if constexpr (DPL <= 8)
    launch_scan<T, DPL, 2>(a, stream);
}

template <typename T>
static void prompts(const DeltaArgs& a, int cpl, hipStream_t stream) {
  const dim3 grid(a.n_tiles, a.G + 2 * a.H);
  // pairs of channels: every head then starts at an even one
  const bool even = a.D % 2 == 0 && a.V % 2 == 0 && a.z_stride % 2 == 0 && a.qkv_stride % 2 == 0;
  auto inputs = even ? delta_inputs_kernel<T, 2> : delta_inputs_kernel<T, 1>;
  inputs<<<grid, 256, 0, stream>>>(a);
  if (a.D <= 16) launch_scan_cols<T, 1>(a, cpl, stream);
  else if (a.D <= 32) launch_scan_cols<T, 2>(a, cpl, stream);
  else if (a.D <= 64) launch_scan_cols<T, 4>(a, cpl, stream);
  else if (a.D <= 128) launch_scan_cols<T, 8>(a, cpl, stream);
  else if (a.D <= 256) launch_scan_cols<T, 16>(a, cpl, stream);
  else if (a.D <= 512) launch_scan_cols<T, 32>(a, cpl, stream);
  else launch_scan_cols<T, 64>(a, cpl, stream);
  const int64_t heads = (int64_t)a.N * a.H;
  delta_output_kernel<T><<<(heads + 3) / 4, 256, 0, stream>>>(a);
}

template <typename T, int VW>
static void step(const DeltaArgs& a, int threads, hipStream_t stream) {
  const int ct = a.V / VW, RG = threads / ct, rows = (a.D + RG - 1) / RG;
  const int bytes = 4 * (3 * a.D + 2 * a.V + 2 * RG * a.V + threads / 64 * 4);
  const dim3 grid(a.H, a.seqs);
  auto k = rows <= 4    ? delta_step_kernel<T, VW, 4>
           : rows <= 8  ? delta_step_kernel<T, VW, 8>
           : rows <= 16 ? delta_step_kernel<T, VW, 16>
                        : delta_step_kernel<T, VW, 0>;
  k<<<grid, threads, bytes, stream>>>(a);
}

extern "C" {

// D, V <= 1024
void launch_delta_prompts(bool bf16, const DeltaArgs* a, int cpl, hipStream_t stream) {
  (bf16 ? prompts<bf16_t> : prompts<float>)(*a, cpl, stream);
}

// V % 4 == 0 or V <= threads
void launch_delta_step(bool bf16, const DeltaArgs* a, int threads, hipStream_t stream) {
  if (a->V % 4 == 0)
    (bf16 ? step<bf16_t, 4> : step<float, 4>)(*a, threads, stream);
  else
    (bf16 ? step<bf16_t, 1> : step<float, 1>)(*a, threads, stream);
}

}  // extern "C"
