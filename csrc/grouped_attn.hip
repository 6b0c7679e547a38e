// Grouped attention over the paged cache, one token per sequence, and the plain kernel
// for every other case (gfx950).
//
// A query at position p sees the keys p - window + 1 .. p and the first ``keep``
// ones, or of those only the ones of its own chunk; scores may be mixed over the heads (the
// plain kernel; talk_attn.hip has the others), capped, get a bias by distance, and a sink
// may join the denominator.  The sink is the softmax's starting state (maximum = sink, sum = 1, no
// value), so that neither the merge of partial sums nor the output knows about it.
// Sigmoid weights need no such state: their partial results are plain sums.
//
// Decode: a workgroup owns one (sequence, key/value head) and up to GM of its query
// heads; its 16 lane groups of 16 take every 16th visible key, a few of them in
// flight, a lane KE dims of the key and VE of the value.  Kept and window keys form one list
// without gaps, so nothing is masked.  Few workgroups split the list (grid.y).
#include "common_t.h"
#include "grouped_attn.h"
#include "latent_attn.h"

#define NEG -1e30f
#define LOG2E 1.44269504088896f

struct KeyList {  // of one query: position of the i-th visible key
  int keep, lo, n;
  DEV int at(int i) const { return i < keep ? i : lo + i - keep; }
};

static DEV KeyList visible_keys(const GroupedArgs& a, int pos) {
  KeyList k;
  k.lo = first_key(a, pos);
  k.keep = min(a.keep, k.lo);
  k.n = k.keep + pos + 1 - k.lo;
  return k;
}

template <int KE, int VE, int GM, bool SIG>
__global__ __launch_bounds__(256, GM * (KE + VE) <= 32 ? 4 : GM * (KE + VE) <= 64 ? 3 : 2) void grouped_decode_kernel(
    const GroupedArgs a) {
  constexpr int D = 16 * KE, V = 16 * VE;
  constexpr int KEYS = GM * (KE + VE) <= 32 ? 4 : 2;  // in flight per lane group
  __shared__ float lds_acc[4][GM][V];
  __shared__ float2 lds_ml[4][GM];
  const int group = a.H / a.G, per = (group + GM - 1) / GM;  // workgroups per kv head
  const int part = blockIdx.x % per;
  const int kvh = blockIdx.x / per % a.G, seq = blockIdx.x / (per * a.G);
  const int h0 = kvh * group + part * GM, heads = min(GM, group - part * GM);
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int j = lane & 15, gid = wid * 4 + (lane >> 4);
  const int64_t row0 = (int64_t)seq * a.H + h0;

  const int pos = a.seq_lens[seq] - 1;
  const KeyList keys = visible_keys(a, pos);
  const int per_split = (keys.n + a.n_split - 1) / a.n_split;
  const int x0 = min(keys.n, (int)blockIdx.y * per_split), x1 = min(keys.n, x0 + per_split);
  if (x0 >= x1) {  // an empty split; those are a row's last ones
    if ((int)threadIdx.x < heads)
      a.part_ml[(int64_t)blockIdx.y * a.rows + row0 + threadIdx.x] = float2{NEG, -1.f};
    return;
  }

  // scores in the exp2 domain: a factor, or c1 - 2 c1 / (exp2(c3 s) + 1)
  const float c1 = a.cap * LOG2E;
  const float mul = a.cap > 0.f ? 2.f * LOG2E * a.scale / a.cap : a.scale * LOG2E;
  float q[GM][KE], m[GM], l[GM], acc[GM][VE];
#pragma unroll
  for (int g = 0; g < GM; ++g) {
    const int h = h0 + min(g, heads - 1);
    const bf16_t* qr = (const bf16_t*)a.q + seq * a.q_stride + (int64_t)h * D + j * KE;
#pragma unroll
    for (int e = 0; e < KE; e += (KE < 8 ? KE : 8)) load_f<(KE < 8 ? KE : 8)>(q[g] + e, qr + e);
    const bool sink = a.sink && blockIdx.y == 0 && gid == 0;
    m[g] = sink ? a.sink[h] * LOG2E : NEG;
    l[g] = sink ? 1.f : 0.f;
#pragma unroll
    for (int e = 0; e < VE; ++e) acc[g][e] = 0.f;
  }

  const int* table = a.tables + (int64_t)seq * a.max_blocks;
  const bf16_t* kc = (const bf16_t*)a.k_cache + kvh * D + j * KE;
  const bf16_t* vc = (const bf16_t*)a.v_cache + kvh * V + j * VE;
  int64_t slot[KEYS];
  auto find = [&](int x) {
#pragma unroll
    for (int u = 0; u < KEYS; ++u) {
      const int k = keys.at(min(x + 16 * u, x1 - 1));
      slot[u] = (int64_t)table[k / a.kv_block] * a.kv_block + k % a.kv_block;
    }
  };
  // biases: distances of n_bias - 1 and more share one
  const int far = a.n_bias - 1;
  float b_far[GM];
#pragma unroll
  for (int g = 0; g < GM; ++g)
    b_far[g] = a.bias ? a.bias[(h0 + min(g, heads - 1)) * a.n_bias + far] * LOG2E : 0.f;
  find(x0 + gid);
  for (int x = x0 + gid; x < x1; x += 16 * KEYS) {
    Pack<bf16_t, KE> k[KEYS];
    Pack<bf16_t, VE> v[KEYS];
#pragma unroll
    for (int u = 0; u < KEYS; ++u) {
      k[u] = *(const Pack<bf16_t, KE>*)(kc + slot[u] * a.G * D);
      v[u] = *(const Pack<bf16_t, VE>*)(vc + slot[u] * a.G * V);
    }
    int dist[KEYS];
    bool near = false;
#pragma unroll
    for (int u = 0; u < KEYS; ++u) {
      dist[u] = pos - keys.at(min(x + 16 * u, x1 - 1));
      near |= dist[u] < far;
    }
    near &= a.bias != nullptr;
    find(x + 16 * KEYS);
#pragma unroll
    for (int g = 0; g < GM; ++g) {
      float s[KEYS], b[KEYS], mt = m[g];
#pragma unroll
      for (int u = 0; u < KEYS; ++u) b[u] = b_far[g];
      if (near) {
        const float* br = a.bias + (int64_t)(h0 + min(g, heads - 1)) * a.n_bias;
#pragma unroll
        for (int u = 0; u < KEYS; ++u) b[u] = br[min(dist[u], far)] * LOG2E;
      }
#pragma unroll
      for (int u = 0; u < KEYS; ++u) {
        float dot = 0.f;
#pragma unroll
        for (int e = 0; e < KE; ++e) dot += q[g][e] * to_f(k[u].v[e]);
        dot = row16_sum(dot) * mul;
        if (a.cap > 0.f)
          dot = c1 - 2.f * c1 * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(dot) + 1.f);
        s[u] = x + 16 * u < x1 ? dot + b[u] : -INFINITY;
        mt = fmaxf(mt, s[u]);
      }
      if constexpr (SIG) {
#pragma unroll
        for (int u = 0; u < KEYS; ++u) {
          const float p = __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-s[u]));
#pragma unroll
          for (int e = 0; e < VE; ++e) acc[g][e] += p * to_f(v[u].v[e]);
        }
        continue;
      }
      const float alpha = __builtin_amdgcn_exp2f(m[g] - mt);
      m[g] = mt;
      l[g] *= alpha;
#pragma unroll
      for (int e = 0; e < VE; ++e) acc[g][e] *= alpha;
#pragma unroll
      for (int u = 0; u < KEYS; ++u) {
        const float p = __builtin_amdgcn_exp2f(s[u] - mt);
        l[g] += p;
#pragma unroll
        for (int e = 0; e < VE; ++e) acc[g][e] += p * to_f(v[u].v[e]);
      }
    }
  }

  // merge the wave's lane groups by shuffles, the waves through LDS
#pragma unroll
  for (int g = 0; g < GM; ++g) {
    float mx = fmaxf(m[g], __shfl_xor(m[g], 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float w = SIG ? 1.f : __builtin_amdgcn_exp2f(m[g] - mx);
    float lg = l[g] * w;
    lg += __shfl_xor(lg, 16, 64);
    lg += __shfl_xor(lg, 32, 64);
#pragma unroll
    for (int e = 0; e < VE; ++e) {
      float o = acc[g][e] * w;
      o += __shfl_xor(o, 16, 64);
      o += __shfl_xor(o, 32, 64);
      if (lane < 16) lds_acc[wid][g][j * VE + e] = o;
    }
    if (lane == 0) lds_ml[wid][g] = float2{mx, lg};
  }
  __syncthreads();
  for (int i = threadIdx.x; i < heads * V; i += 256) {
    const int g = i / V, e = i % V;
    float mx = NEG, sum = 0.f, o = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) mx = fmaxf(mx, lds_ml[w][g].x);
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float f = SIG ? 1.f : __builtin_amdgcn_exp2f(lds_ml[w][g].x - mx);
      sum += f * lds_ml[w][g].y;
      o += f * lds_acc[w][g][e];
    }
    if (a.n_split == 1) {
      if (!SIG) o /= sum;
      if (a.gate) o *= sigmoid_f(bf2f(((const bf16_t*)a.gate)[seq * a.gate_stride + h0 + g]));
      ((bf16_t*)a.out)[seq * a.out_stride + (int64_t)(h0 + g) * V + e] = from_f<bf16_t>(o);
    } else {
      const int64_t at = (int64_t)blockIdx.y * a.rows + row0 + g;
      a.part[at * V + e] = o;
      if (e == 0) a.part_ml[at] = SIG ? float2{0.f, 1.f} : float2{mx, sum};
    }
  }
}

// Any dtype and size: a workgroup per (token, head), its 4 waves stride over the keys,
// a lane holds every 64th dim.
template <typename T, int NE>
__global__ __launch_bounds__(256) void grouped_plain_kernel(
    const GroupedArgs a, const int d, const int v) {
  const int h = blockIdx.y, kvh = h / (a.H / a.G);
  int seq, pos, token;
  if (a.tile_seq) {
    seq = a.tile_seq[blockIdx.x];
    pos = a.ctx_lens[seq] + a.tile_q0[blockIdx.x];
    token = a.row_starts[seq] + a.tile_q0[blockIdx.x];
  } else {
    seq = token = blockIdx.x;
    pos = a.seq_lens[seq] - 1;
  }
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int* table = a.tables + (int64_t)seq * a.max_blocks;
  const T* qr = (const T*)a.q + token * a.q_stride;
  float q[NE], acc[NE] = {};
  // mixed scores are those of one long query, the mix of the heads that share a key head,
  // against all key heads
  const int dk = a.talk ? a.G * d : d, k_at = a.talk ? 0 : kvh * d, group = a.H / a.G;
#pragma unroll
  for (int e = 0; e < NE; ++e) {
    const int i = e * 64 + lane;
    q[e] = 0.f;
    if (i >= dk) continue;
    if (a.talk) {
      const int g0 = i / d * group;
      for (int g = g0; g < g0 + group; ++g)
        q[e] += a.talk[h * a.H + g] * to_f(qr[(int64_t)g * d + i % d]);
    } else {
      q[e] = to_f(qr[(int64_t)h * d + i]);
    }
  }
  const bool sink = a.sink && wid == 0;
  float m = sink ? a.sink[h] : NEG, l = sink ? 1.f : 0.f;
  const KeyList keys = visible_keys(a, pos);
  for (int x = wid; x < keys.n; x += 4) {
    const int k = keys.at(x);
    const int64_t slot = (int64_t)table[k / a.kv_block] * a.kv_block + k % a.kv_block;
    const T* kr = (const T*)a.k_cache + slot * a.G * d + k_at;
    const T* vr = (const T*)a.v_cache + (slot * a.G + kvh) * v;
    float dot = 0.f, val[NE];
#pragma unroll
    for (int e = 0; e < NE; ++e) {
      const int i = e * 64 + lane;
      if (i < dk) dot += q[e] * to_f(kr[i]);
      val[e] = i < v ? to_f(vr[i]) : 0.f;
    }
    dot = wave_sum(dot) * a.scale;
    if (a.cap > 0.f) dot = a.cap * tanhf(dot / a.cap);
    if (a.bias) dot += a.bias[(int64_t)h * a.n_bias + min(pos - k, a.n_bias - 1)];
    if (a.sigmoid) {
      const float p = 1.f / (1.f + expf(-dot));
#pragma unroll
      for (int e = 0; e < NE; ++e) acc[e] += p * val[e];
      continue;
    }
    const float mn = fmaxf(m, dot);
    const float alpha = expf(m - mn), p = expf(dot - mn);
    m = mn;
    l = l * alpha + p;
#pragma unroll
    for (int e = 0; e < NE; ++e) acc[e] = acc[e] * alpha + p * val[e];
  }
  __shared__ float part[4][NE * 64];
  __shared__ float2 ml[4];
#pragma unroll
  for (int e = 0; e < NE; ++e) part[wid][e * 64 + lane] = acc[e];
  if (lane == 0) ml[wid] = float2{m, l};
  __syncthreads();
  float mx = NEG, w[4], sum = 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) mx = fmaxf(mx, ml[i].x);
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    w[i] = a.sigmoid ? 1.f : expf(ml[i].x - mx);
    sum += w[i] * ml[i].y;
  }
  float f = a.sigmoid ? 1.f : 1.f / sum;
  if (a.gate) f *= sigmoid_f(to_f(((const T*)a.gate)[token * a.gate_stride + h]));
  for (int i = threadIdx.x; i < v; i += 256) {
    float o = 0.f;
#pragma unroll
    for (int n = 0; n < 4; ++n) o += w[n] * part[n][i];
    ((T*)a.out)[token * a.out_stride + (int64_t)h * v + i] = from_f<T>(o * f);
  }
}

// k [n, G, d] and v [n, G, v] rows into their slots, 16 bytes a thread.
__global__ __launch_bounds__(256) void cache_keys_values_kernel(
    ulonglong2* __restrict__ k_cache, ulonglong2* __restrict__ v_cache,
    const ulonglong2* __restrict__ k, const ulonglong2* __restrict__ v,
    const int64_t* __restrict__ slots, const int k_units, const int v_units,
    const int64_t stride, const int64_t total) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  const int units = k_units + v_units;
  const int64_t n = i / units;
  const int u = (int)(i - n * units);
  if (u < k_units)
    k_cache[slots[n] * k_units + u] = k[n * stride + u];
  else
    v_cache[slots[n] * v_units + u - k_units] = v[n * stride + u - k_units];
}

template <int KE, int VE, bool SIG>
static void launch_decode(const GroupedArgs& a, int seqs, int gm, hipStream_t stream) {
  if (KE + VE > 16 && gm > 4) gm = 4;
  const int group = a.H / a.G;
  const dim3 grid(seqs * a.G * ((group + gm - 1) / gm), a.n_split);
  if (gm == 1)
    grouped_decode_kernel<KE, VE, 1, SIG><<<grid, 256, 0, stream>>>(a);
  else if (gm == 2)
    grouped_decode_kernel<KE, VE, 2, SIG><<<grid, 256, 0, stream>>>(a);
  else if (gm == 4)
    grouped_decode_kernel<KE, VE, 4, SIG><<<grid, 256, 0, stream>>>(a);
  else if constexpr (KE + VE <= 16)
    grouped_decode_kernel<KE, VE, 8, SIG><<<grid, 256, 0, stream>>>(a);
}

template <int KE, int VE>
static bool launch_decode(const GroupedArgs& a, int seqs, int gm, hipStream_t stream) {
  (a.sigmoid ? launch_decode<KE, VE, true> : launch_decode<KE, VE, false>)(a, seqs, gm, stream);
  return true;
}

template <int KE>
static bool launch_decode_v(const GroupedArgs& a, int v, int seqs, int gm,
                            hipStream_t stream) {
  switch (v) {
    case 64: return launch_decode<KE, 4>(a, seqs, gm, stream);
    case 128: return launch_decode<KE, 8>(a, seqs, gm, stream);
    case 256: return launch_decode<KE, 16>(a, seqs, gm, stream);
    default: return false;
  }
}

template <typename T>
static bool launch_plain(const GroupedArgs& a, int d, int v, int tokens, hipStream_t stream) {
  const int dk = a.talk ? a.G * d : d;
  const int ne = ((dk > v ? dk : v) + 63) / 64;
  if (ne > 64) return false;
  auto k = ne <= 1    ? grouped_plain_kernel<T, 1>
           : ne <= 2  ? grouped_plain_kernel<T, 2>
           : ne <= 4  ? grouped_plain_kernel<T, 4>
           : ne <= 8  ? grouped_plain_kernel<T, 8>
           : ne <= 32 ? grouped_plain_kernel<T, 32>
                      : grouped_plain_kernel<T, 64>;
  k<<<dim3(tokens, a.H), 256, 0, stream>>>(a, d, v);
  return true;
}

extern "C" {

// gm: query heads of one key/value head per workgroup, 1, 2, 4 or 8 (8 if d + v <= 256)
bool launch_grouped_decode(const GroupedArgs* a, int d, int v, int seqs, int gm,
                           hipStream_t stream) {
  bool ok = false;
  switch (d) {
    case 64: ok = launch_decode_v<4>(*a, v, seqs, gm, stream); break;
    case 128: ok = launch_decode_v<8>(*a, v, seqs, gm, stream); break;
    case 256: ok = launch_decode_v<16>(*a, v, seqs, gm, stream); break;
  }
  if (ok && a->n_split > 1) {
    const SplitOut out = {a->out, a->gate, a->out_stride, a->gate_stride, a->H, a->sigmoid};
    launch_split_combine(&out, a->part, a->part_ml, a->rows, v, a->n_split, stream);
  }
  return ok;
}

bool launch_grouped_plain(bool bf16, const GroupedArgs* a, int d, int v, int tokens,
                          hipStream_t stream) {
  return (bf16 ? launch_plain<bf16_t> : launch_plain<float>)(*a, d, v, tokens, stream);
}

void launch_cache_keys_values(void* k_cache, void* v_cache, const void* k, const void* v,
                              const int64_t* slots, int k_units, int v_units, int64_t stride,
                              int n, hipStream_t stream) {
  const int64_t total = (int64_t)n * (k_units + v_units);
  cache_keys_values_kernel<<<(total + 255) / 256, 256, 0, stream>>>(
      (ulonglong2*)k_cache, (ulonglong2*)v_cache, (const ulonglong2*)k,
      (const ulonglong2*)v, slots, k_units, v_units, stride, total);
}

}  // extern "C"
