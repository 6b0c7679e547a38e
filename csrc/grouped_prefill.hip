// Grouped attention of prompt portions over the paged cache on the matrix cores
// (gfx950): windows that keep the first tokens, chunks, capped scores, biases by distance, a
// sink; softmax or sigmoid weights; a gate per head.
//
// A workgroup owns 128 query rows of one head, a wave 32 of them.  Keys and values
// stream through LDS in tiles of 64, double buffered, loaded straight from their pages;
// LDS rows are 16-byte units XOR-swizzled on the source address.  The tiles are those
// of the kept tokens and those of the window; what lies between is never read.
//
//   QK^T (A = keys, B = queries, 32x32x16): a lane owns one query and, per 32
//     keys, the rows (r & 3) + 8 (r >> 2) + 4 (lane >> 5)
//   softmax: 32 registers and one exchange between the lane halves; it starts from
//     the sink (maximum = sink, sum = 1).  Sigmoid weights need neither
//   biases: beyond the last distance with one of its own they are one number a head;
//     only tiles nearer than that look them up
//   PV (A = values^T, B = probabilities): the product's 16 key slots are taken in
//     the order the scores already have, so the probabilities never leave their lane;
//     the value fragments are read transposed (ds_read_b64_tr_b16) in that order
//
// Tiles come heaviest first; the query heads of one key/value head stay on one XCD.
#include "common_t.h"
#include "grouped_attn.h"

typedef __bf16 bf16x8_v __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4_v __attribute__((ext_vector_type(4)));
typedef float f32x16_v __attribute__((ext_vector_type(16)));
typedef __attribute__((address_space(3))) char lds_char;
typedef __attribute__((address_space(3))) bf16x4_v lds_bf16x4;
typedef __attribute__((address_space(1))) const char glob_char;

#define KT 64
#define QROWS 128
#define NEG -1e30f
#define LOG2E 1.44269504088896f

// FORM: 0 softmax, 1 softmax of capped scores, 2 sigmoid
template <int DN, int VN, int FORM>
__global__ __launch_bounds__(256, DN + VN <= 4 ? 2 : 1) void grouped_prefill_kernel(
    const GroupedArgs a) {
  constexpr bool CAP = FORM == 1, SIG = FORM == 2;
  constexpr int D = 64 * DN, V = 64 * VN;
  constexpr int KU = D / 8, VU = V / 8;       // units per LDS row
  constexpr int STEPS = D / 16, VT = V / 32;
  constexpr int K_BYTES = KT * D * 2, TILE_BYTES = K_BYTES + KT * V * 2;
  extern __shared__ char lds[];
  int* const slots = (int*)(lds + 2 * TILE_BYTES);  // [2][KT]

  // 8 XCDs take consecutive workgroups in turn: give each its own run of heads
  int head, tile;
  {
    const int id = blockIdx.x;
    if (a.H % 8 == 0) {
      const int per = a.H / 8, slot = id >> 3;
      head = (id & 7) * per + slot % per;
      tile = slot / per;
    } else {
      head = id % a.H;
      tile = id / a.H;
    }
    tile = a.n_tiles - 1 - tile;
  }
  const int kvh = head / (a.H / a.G);
  const int seq = a.tile_seq[tile], q0 = a.tile_q0[tile];
  const int ctx = a.ctx_lens[seq];
  const int rows = min(QROWS, a.seq_lens[seq] - ctx - q0);
  const int64_t row0 = a.row_starts[seq] + q0;
  const int* table = a.tables + (int64_t)seq * a.max_blocks;

  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int c = lane & 31, half = lane >> 5;
  const int r = wid * 32 + c;
  const bool live = r < rows;
  const int qpos = live ? ctx + q0 + r : -1;

  // key tiles: those with kept tokens, then those some row's window reaches
  const int k_end = ctx + q0 + rows;
  const int kept = (min(a.keep, k_end) + KT - 1) / KT;
  const int first = max(kept, first_key(a, ctx + q0) / KT);
  const int n_tiles = kept + max(0, (k_end + KT - 1) / KT - first);
  auto key_of = [&](int t) { return (t < kept ? t : first + t - kept) * KT; };
  // this thread's key of tile t, as a slot
  auto find_slot = [&](int t) {
    const int k = min(key_of(t) + lane, k_end - 1);
    return table[k / a.kv_block] * a.kv_block + k % a.kv_block;
  };
  const bf16_t* kp = (const bf16_t*)a.k_cache + (int64_t)kvh * D;
  const bf16_t* vp = (const bf16_t*)a.v_cache + (int64_t)kvh * V;

  auto stage = [&](int t) {
    char* dst = lds + (t & 1) * TILE_BYTES;
    const int* sl = slots + (t & 1) * KT;
#pragma unroll
    for (int i = 0; i < KU / 4; ++i) {
      const int piece = i * 4 + wid;
      const int u = piece * 64 + lane;
      const int key = u / KU;
      const int unit = (u - key * KU) ^ (((key & 3) << 1) | ((key >> 2) & 1));
      __builtin_amdgcn_global_load_lds(
          (glob_char*)(kp + (int64_t)sl[key] * a.G * D + unit * 8),
          (lds_char*)(dst + piece * 1024), 16, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < VU / 4; ++i) {
      const int piece = i * 4 + wid;
      const int u = piece * 64 + lane;
      const int key = u / VU;
      const int unit = (u - key * VU) ^ (((key & 3) << 1) | ((key >> 2) & 1));
      __builtin_amdgcn_global_load_lds(
          (glob_char*)(vp + (int64_t)sl[key] * a.G * V + unit * 8),
          (lds_char*)(dst + K_BYTES + piece * 1024), 16, 0, 0);
    }
  };
  if (wid < 2 && wid < n_tiles) slots[wid * KT + lane] = find_slot(wid);
  __syncthreads();
  stage(0);

  // query fragments: 8 consecutive dims of row c per step
  bf16x8_v qf[STEPS];
  {
    const int64_t n = row0 + (live ? r : 0);
    const bf16_t* qr = (const bf16_t*)a.q + n * a.q_stride + (int64_t)head * D + half * 8;
#pragma unroll
    for (int s = 0; s < STEPS; ++s) qf[s] = *(const bf16x8_v*)(qr + s * 16);
  }

  // scores in the exp2 domain: a factor, or c1 - 2 c1 / (exp2(c3 s) + 1)
  const float c1 = a.cap * LOG2E;
  const float mul = CAP ? 2.f * LOG2E * a.scale / a.cap : a.scale * LOG2E;
  float m_run = a.sink ? a.sink[head] * LOG2E : NEG;
  float l_run = a.sink && half == 0 ? 1.f : 0.f;
  const float* bias = a.bias ? a.bias + (int64_t)head * a.n_bias : nullptr;
  const int far = a.n_bias - 1;
  const float b_far = bias ? bias[far] * LOG2E : 0.f;
  f32x16_v o[VT] = {};
  const int w_lo = ctx + q0 + wid * 32;                    // wave's positions
  const int w_hi = min(w_lo + 31, k_end - 1);
  const int lo = live ? first_key(a, qpos) : 0;
  const int lo_lo = first_key(a, w_lo), lo_hi = first_key(a, max(w_lo, w_hi));
  const int sw_k = ((c & 3) << 1) | ((c >> 2) & 1);
  const int i16 = lane & 15, g = lane >> 4;

  for (int t = 0; t < n_tiles; ++t) {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();  // tile t landed for every wave; tile t-1 is fully read
    // a slot for tile t + 2, looked up ahead of the tile's loads
    int next = 0;
    const bool look = wid == 0 && t + 2 < n_tiles;
    if (look) next = find_slot(t + 2);
    if (t + 1 < n_tiles) stage(t + 1);
    const int key0 = key_of(t);
    // a tile that one of this wave's rows sees
    if (wid * 32 < rows && key0 <= w_hi && (key0 + KT - 1 >= lo_lo || key0 < a.keep)) {
      const char* kt = lds + (t & 1) * TILE_BYTES;
      f32x16_v s[2] = {};
#pragma unroll
      for (int st = 0; st < STEPS; ++st) {
        const int off = ((st * 2 + half) ^ sw_k) << 4;
#pragma unroll
        for (int b = 0; b < 2; ++b) {
          const bf16x8_v kf = *(const bf16x8_v*)(kt + (b * 32 + c) * (D * 2) + off);
          s[b] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qf[st], s[b], 0, 0, 0);
        }
      }
      const bool edge = key0 + KT - 1 > w_lo || key0 < lo_hi;
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int e = 0; e < 16; ++e) {
          float v = s[b][e] * mul;
          if (CAP) v = c1 - 2.f * c1 * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(v) + 1.f);
          s[b][e] = v + b_far;
        }
      if (bias && w_lo - (key0 + KT - 1) < far) {
#pragma unroll
        for (int b = 0; b < 2; ++b)
#pragma unroll
          for (int e = 0; e < 16; ++e) {
            const int key = key0 + b * 32 + (e & 3) + 8 * (e >> 2) + 4 * half;
            s[b][e] += bias[min(max(qpos - key, 0), far)] * LOG2E - b_far;
          }
      }
      float mt = NEG;
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int e = 0; e < 16; ++e) {
          if (edge) {
            const int key = key0 + b * 32 + (e & 3) + 8 * (e >> 2) + 4 * half;
            if (key > qpos || (key < lo && key >= a.keep)) s[b][e] = -INFINITY;
          }
          mt = fmaxf(mt, s[b][e]);
        }
      if constexpr (SIG) {
#pragma unroll
        for (int b = 0; b < 2; ++b)
#pragma unroll
          for (int e = 0; e < 16; ++e)
            s[b][e] = __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-s[b][e]));
      } else {
        mt = fmaxf(mt, __shfl_xor(mt, 32, 64));
        if (__any(mt > m_run)) {
          const float m_new = fmaxf(m_run, mt);
          const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
          m_run = m_new;
          l_run *= alpha;
#pragma unroll
          for (int n = 0; n < VT; ++n) o[n] *= alpha;
        }
        float sum = 0.f;
#pragma unroll
        for (int b = 0; b < 2; ++b)
#pragma unroll
          for (int e = 0; e < 16; ++e) {
            s[b][e] = __builtin_amdgcn_exp2f(s[b][e] - m_run);
            sum += s[b][e];
          }
        l_run += sum;
      }

      const char* vt = kt + K_BYTES;
#pragma unroll
      for (int ks = 0; ks < 4; ++ks) {
        bf16x8_v pf;
#pragma unroll
        for (int e = 0; e < 8; ++e) pf[e] = (__bf16)s[ks >> 1][(ks & 1) * 8 + e];
        const int key = ks * 16 + 4 * (g >> 1) + (i16 >> 2);
        const int sw = ((i16 >> 2) << 1) | (g >> 1);
        const char* vrow = vt + key * (V * 2) + (i16 & 1) * 8;
#pragma unroll
        for (int n = 0; n < VT; ++n) {
          const int off = ((n * 4 + (g & 1) * 2 + ((i16 & 3) >> 1)) ^ sw) << 4;
          const bf16x4_v lo =
              __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds_bf16x4*)(vrow + off));
          const bf16x4_v hi =
              __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds_bf16x4*)(vrow + 8 * (V * 2) + off));
          const bf16x8_v vf = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
          o[n] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, pf, o[n], 0, 0, 0);
        }
      }
    }
    // tile t's slots were consumed by its stage, before this iteration's barrier
    if (look) slots[(t & 1) * KT + lane] = next;
  }

  l_run += __shfl_xor(l_run, 32, 64);
  if (!live) return;
  float inv = SIG ? 1.f : l_run > 0.f ? 1.f / l_run : 0.f;
  if (a.gate) inv *= sigmoid_f(bf2f(((const bf16_t*)a.gate)[(row0 + r) * a.gate_stride + head]));
  bf16_t* dst = (bf16_t*)a.out + (row0 + r) * a.out_stride + (int64_t)head * V + 4 * half;
#pragma unroll
  for (int t = 0; t < VT; ++t)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float v[4] = {o[t][4 * e] * inv, o[t][4 * e + 1] * inv, o[t][4 * e + 2] * inv,
                          o[t][4 * e + 3] * inv};
      store_f<4>(dst + t * 32 + e * 8, v);
    }
}

template <int DN, int VN, int FORM>
static void launch(const GroupedArgs& a, hipStream_t stream) {
  constexpr int bytes = 2 * KT * (64 * DN + 64 * VN) * 2 + 2 * KT * 4;
  static_assert(bytes <= 160 * 1024, "LDS");
  static bool attr_set = false;
  if (!attr_set) {
    (void)hipFuncSetAttribute((const void*)grouped_prefill_kernel<DN, VN, FORM>,
                              hipFuncAttributeMaxDynamicSharedMemorySize, bytes);
    attr_set = true;
  }
  grouped_prefill_kernel<DN, VN, FORM><<<a.n_tiles * a.H, 256, bytes, stream>>>(a);
}

template <int DN, int VN>
static bool launch_form(const GroupedArgs& a, hipStream_t stream) {
  if (a.sigmoid && a.cap > 0.f) return false;
  (a.sigmoid       ? launch<DN, VN, 2>
   : a.cap > 0.f   ? launch<DN, VN, 1>
                   : launch<DN, VN, 0>)(a, stream);
  return true;
}

template <int DN>
static bool launch_v(const GroupedArgs& a, int v, hipStream_t stream) {
  switch (v) {
    case 64: return launch_form<DN, 1>(a, stream);
    case 128: return launch_form<DN, 2>(a, stream);
    case 256: return launch_form<DN, 4>(a, stream);
    default: return false;
  }
}

extern "C" bool launch_grouped_prefill(const GroupedArgs* a, int d, int v,
                                       hipStream_t stream) {
  switch (d) {
    case 64: return launch_v<1>(*a, v, stream);
    case 128: return launch_v<2>(*a, v, stream);
    case 256: return launch_v<4>(*a, v, stream);
    default: return false;
  }
}
