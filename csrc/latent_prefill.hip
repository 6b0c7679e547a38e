// Prompt attention over keys and values expanded from latents (gfx950).
//
// A workgroup owns 128 query rows of one head, a wave 32 of them.  Keys and
// values stream through LDS in tiles of 64, double buffered, loaded straight
// from global memory; LDS rows are 16-byte units XOR-swizzled on the source
// address.  Everything but the tile hand-over is lane-local:
//
//   QK^T (A = keys, B = queries, 32x32x16): a lane owns one query and, per 32
//     keys, the rows (r & 3) + 8 (r >> 2) + 4 (lane >> 5)
//   softmax: 32 registers and one exchange between the lane halves
//   PV (A = values^T, B = probabilities): the product's 16 key slots are taken in
//     the order the scores already have, half 0 holding keys 0-3 and 8-11 and
//     half 1 keys 4-7 and 12-15, so the probabilities never leave their lane; the
//     value fragments are read transposed (ds_read_b64_tr_b16) in that order
//
// A key is [dim | 64 rotated]: the first part per head, the second shared by the
// heads.  Queries are rotated as they are loaded; the head gate is applied as the
// output is stored.  Tiles come heaviest first, and the heads of one XCD's
// workgroups stay together so that their keys share its L2.
#include "common_t.h"
#include "latent_attn.h"

typedef __bf16 bf16x8_v __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4_v __attribute__((ext_vector_type(4)));
typedef float f32x16_v __attribute__((ext_vector_type(16)));
typedef __attribute__((address_space(3))) char lds_char;
typedef __attribute__((address_space(3))) bf16x4_v lds_bf16x4;
typedef __attribute__((address_space(1))) const char glob_char;

#define KT 64
#define ROT 64
#define QROWS 128
#define NEG -1e30f

template <int DN, int VN>
__global__ __launch_bounds__(256, DN + VN <= 4 ? 2 : 1) void latent_prefill_kernel(
    const LatentPrefillArgs a) {
  constexpr int D = 64 * DN, V = 64 * VN, QK = D + ROT;
  constexpr int KU = QK / 8, VU = V / 8;       // units per LDS row
  constexpr int STEPS = QK / 16, VT = V / 32;
  constexpr int K_BYTES = KT * QK * 2, TILE_BYTES = K_BYTES + KT * V * 2;
  extern __shared__ char lds[];

  // 8 XCDs take consecutive workgroups in turn: give each its own heads
  int head, tile;
  {
    const int id = blockIdx.x;
    if (a.H % 8 == 0) {
      const int per = a.H / 8, slot = id >> 3;
      head = (slot % per) * 8 + (id & 7);
      tile = slot / per;
    } else {
      head = id % a.H;
      tile = id / a.H;
    }
    tile = a.n_tiles - 1 - tile;
  }
  const int seq = a.tile_seq[tile], q0 = a.tile_q0[tile];
  const int ctx = a.ctx_lens[seq];
  const int rows = min(QROWS, a.seq_lens[seq] - ctx - q0);
  const int64_t row0 = a.row_starts[seq] + q0;

  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int c = lane & 31, half = lane >> 5;
  const int r = wid * 32 + c;
  const bool live = r < rows;
  const int qpos = live ? ctx + q0 + r : -1;

  // this tile's keys, as rows of the expanded buffer
  const int first = a.key_first[seq];           // position of the sequence's first row
  const int k_begin = max(first, ctx + q0 - a.window + 1);
  const int k_end = ctx + q0 + rows;
  const int n_tiles = (k_end - k_begin + KT - 1) / KT;
  const int64_t kbuf = (int64_t)a.key_starts[seq] + (k_begin - first);
  const bf16_t* kp = (const bf16_t*)a.kv + kbuf * a.kv_stride + (int64_t)head * D;
  const bf16_t* vp = (const bf16_t*)a.kv + kbuf * a.kv_stride + (int64_t)a.H * D +
                     (int64_t)head * V;
  const bf16_t* rp = (const bf16_t*)a.k_rot + kbuf * a.rot_stride;
  const int k_last = k_end - k_begin - 1;

  auto stage = [&](int t) {
    char* dst = lds + (t & 1) * TILE_BYTES;
#pragma unroll
    for (int i = 0; i < KU / 4; ++i) {
      const int piece = i * 4 + wid;
      const int u = piece * 64 + lane;
      const int key = u / KU;
      const int unit = (u - key * KU) ^ (((key & 3) << 1) | ((key >> 2) & 1));
      const int64_t k = min(t * KT + key, k_last);
      const bf16_t* src =
          unit < D / 8 ? kp + k * a.kv_stride + unit * 8 : rp + k * a.rot_stride + unit * 8 - D;
      __builtin_amdgcn_global_load_lds((glob_char*)src, (lds_char*)(dst + piece * 1024),
                                       16, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < VU / 4; ++i) {
      const int piece = i * 4 + wid;
      const int u = piece * 64 + lane;
      const int key = u / VU;
      const int unit = (u - key * VU) ^ (((key & 3) << 1) | ((key >> 2) & 1));
      const int64_t k = min(t * KT + key, k_last);
      __builtin_amdgcn_global_load_lds((glob_char*)(vp + k * a.kv_stride + unit * 8),
                                       (lds_char*)(dst + K_BYTES + piece * 1024), 16, 0, 0);
    }
  };
  stage(0);

  // query fragments: 8 consecutive dims of row c per step
  bf16x8_v qf[STEPS];
  {
    const int64_t n = row0 + (live ? r : 0);
    const bf16_t* qr = (const bf16_t*)a.q + n * a.q_stride + (int64_t)head * QK + half * 8;
#pragma unroll
    for (int s = 0; s < STEPS; ++s) qf[s] = *(const bf16x8_v*)(qr + s * 16);
    const int pairs = a.rot_dim >> 1;
    const float* ct = a.cos_sin + (int64_t)max(qpos, 0) * pairs;
    const float* st = ct + a.positions * pairs;
#pragma unroll
    for (int s = D / 16; s < STEPS; ++s)
#pragma unroll
      for (int p = 0; p < 4; ++p) {
        // padding is zero: any angle
        const int i = min((s * 16 - D + half * 8) / 2 + p, pairs - 1);
        const float x = (float)qf[s][2 * p], y = (float)qf[s][2 * p + 1];
        qf[s][2 * p] = (__bf16)(x * ct[i] - y * st[i]);
        qf[s][2 * p + 1] = (__bf16)(y * ct[i] + x * st[i]);
      }
  }

  const float scale2 = a.scale * 1.44269504088896f;
  // a sink is the softmax's starting state: its maximum, one term of the sum, no value
  float m_run = a.sink ? a.sink[head] * 1.44269504088896f : NEG;
  float l_run = a.sink && half == 0 ? 1.f : 0.f;
  f32x16_v o[VT] = {};
  const int w_lo = ctx + q0 + wid * 32;                    // wave's positions
  const int w_hi = min(w_lo + 31, ctx + q0 + rows - 1);
  const int sw_k = ((c & 3) << 1) | ((c >> 2) & 1);
  const int i16 = lane & 15, g = lane >> 4;

  for (int t = 0; t < n_tiles; ++t) {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();  // tile t landed for every wave; tile t-1 is fully read
    if (t + 1 < n_tiles) stage(t + 1);
    const int key0 = k_begin + t * KT;
    // tiles none of this wave's rows see
    if (key0 > w_hi || w_lo - (key0 + KT - 1) >= a.window) continue;
    const char* kt = lds + (t & 1) * TILE_BYTES;

    f32x16_v s[2] = {};
#pragma unroll
    for (int st = 0; st < STEPS; ++st) {
      const int off = ((st * 2 + half) ^ sw_k) << 4;
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        const bf16x8_v kf = *(const bf16x8_v*)(kt + (b * 32 + c) * (QK * 2) + off);
        s[b] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qf[st], s[b], 0, 0, 0);
      }
    }
    const bool edge = key0 + KT - 1 > w_lo || w_hi - key0 >= a.window;
    float mt = NEG;
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int e = 0; e < 16; ++e) {
        float v = s[b][e] * scale2;
        if (edge) {
          const int key = key0 + b * 32 + (e & 3) + 8 * (e >> 2) + 4 * half;
          if (key > qpos || qpos - key >= a.window) v = -INFINITY;
        }
        s[b][e] = v;
        mt = fmaxf(mt, v);
      }
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

  l_run += __shfl_xor(l_run, 32, 64);
  if (!live) return;
  const int64_t n = row0 + r;
  float inv = l_run > 0.f ? 1.f / l_run : 0.f;
  if (a.gate) inv *= sigmoid_f(bf2f(((const bf16_t*)a.gate)[n * a.gate_stride + head]));
  bf16_t* dst = (bf16_t*)a.out + n * a.out_stride + (int64_t)head * V + 4 * half;
#pragma unroll
  for (int t = 0; t < VT; ++t)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float v[4] = {o[t][4 * e] * inv, o[t][4 * e + 1] * inv, o[t][4 * e + 2] * inv,
                          o[t][4 * e + 3] * inv};
      store_f<4>(dst + t * 32 + e * 8, v);
    }
}

// out[starts[s] + i] = the cached row of position first[s] + i; a wave per row,
// 16 bytes a lane.
__global__ __launch_bounds__(256) void latent_gather_kernel(
    bf16_t* __restrict__ out, const bf16_t* __restrict__ cache,
    const int* __restrict__ tables, const int* __restrict__ seq_lens,
    const int* __restrict__ first, const int* __restrict__ starts, const int row,
    const int max_blocks, const int kv_block) {
  const int seq = blockIdx.y;
  const int pos = first[seq] + blockIdx.x * 4 + (threadIdx.x >> 6);
  if (pos >= seq_lens[seq]) return;
  const int64_t slot =
      (int64_t)tables[(int64_t)seq * max_blocks + pos / kv_block] * kv_block + pos % kv_block;
  const bf16_t* src = cache + slot * row;
  bf16_t* dst = out + (int64_t)(starts[seq] + pos - first[seq]) * row;
  for (int i = (threadIdx.x & 63) * 8; i < row; i += 512)
    *(ulonglong2*)(dst + i) = *(const ulonglong2*)(src + i);
}

template <int DN, int VN>
static void launch(const LatentPrefillArgs& a, hipStream_t stream) {
  constexpr int bytes = 2 * KT * (64 * DN + ROT + 64 * VN) * 2;
  static_assert(bytes <= 160 * 1024, "LDS");
  static bool attr_set = false;
  if (!attr_set) {
    (void)hipFuncSetAttribute((const void*)latent_prefill_kernel<DN, VN>,
                              hipFuncAttributeMaxDynamicSharedMemorySize, bytes);
    attr_set = true;
  }
  latent_prefill_kernel<DN, VN><<<a.n_tiles * a.H, 256, bytes, stream>>>(a);
}

template <int DN>
static bool launch_v(const LatentPrefillArgs& a, int v, hipStream_t stream) {
  switch (v) {
    case 64: launch<DN, 1>(a, stream); return true;
    case 128: launch<DN, 2>(a, stream); return true;
    case 256: launch<DN, 4>(a, stream); return true;
    default: return false;
  }
}

extern "C" {

bool launch_latent_prefill(const LatentPrefillArgs* a, int d, int v, hipStream_t stream) {
  switch (d) {
    case 64: return launch_v<1>(*a, v, stream);
    case 128: return launch_v<2>(*a, v, stream);
    case 256: return launch_v<4>(*a, v, stream);
    default: return false;
  }
}

void launch_latent_gather(void* out, const void* cache, const int* tables,
                          const int* seq_lens, const int* first, const int* starts, int seqs,
                          int max_keys, int row, int max_blocks, int kv_block,
                          hipStream_t stream) {
  latent_gather_kernel<<<dim3((max_keys + 3) / 4, seqs), 256, 0, stream>>>(
      (bf16_t*)out, (const bf16_t*)cache, tables, seq_lens, first, starts, row, max_blocks,
      kv_block);
}

}  // extern "C"
