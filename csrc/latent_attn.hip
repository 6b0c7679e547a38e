// Attention of absorbed queries over cached latent rows (gfx950).
//
// A cached row [latent: rank | rotated: 64] is the key of every head, and its
// latent part is the value of every head: one row serves all heads' products
// twice.  Queries are flattened (token, head) rows; a workgroup owns 16*MG of
// them, which for decode are the heads of one sequence.
//
//   tile = 64 keys staged once in LDS by direct global->LDS loads (row-major,
//     16-byte units XOR-swizzled on the source address), double buffered
//   QK^T: wave w takes keys 16w..16w+15, all query rows (A = keys, B = queries,
//     so a lane owns one query row and 4 of its keys)
//   softmax: row maxima cross waves through LDS, probabilities go to LDS as bf16
//   PV: wave w takes latent columns [w*rank/4, ...) for all 64 keys; the value
//     fragments are the same LDS tile read transposed (ds_read_b64_tr_b16)
//
// So each wave reads half of the tile once per product, whatever MG is, and the
// accumulator of a wave is rank/4 columns only.  The swizzle moves 4 consecutive
// keys by 2 units each, which keeps both the row reads (16 keys, one unit) and
// the transposed reads (4 keys, two units) off each other's banks.
//
// Keys past a sequence's end are clamped to its last key and masked; split-K
// partials are merged by split_combine_kernel.  The grid depends on host
// values only (capture-safe); lengths are read on the device.
#include "common_t.h"
#include "latent_attn.h"

typedef __bf16 bf16x8_v __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4_v __attribute__((ext_vector_type(4)));
typedef float f32x4_v __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) char lds_char;
typedef __attribute__((address_space(3))) bf16x4_v lds_bf16x4;
typedef __attribute__((address_space(1))) const char glob_char;

#define KT 64          // keys per tile
#define ROT 64         // padded rotated dims
#define NEG -1e30f
#define PPAD 72        // probability row in LDS, bf16 elements

// one query tile's place
struct Tile {
  int seq, r0, count, ctx, S, token0;
};

static DEV Tile find_tile(const LatentArgs& a, int rows_per_tile) {
  Tile t;
  if (a.tile_seq) {
    t.seq = a.tile_seq[blockIdx.x];
    t.r0 = a.tile_r0[blockIdx.x];
    t.S = a.seq_lens[t.seq];
    t.ctx = a.ctx_lens[t.seq];
    t.token0 = a.row_starts[t.seq];
  } else {
    const int per_seq = (a.H + rows_per_tile - 1) / rows_per_tile;
    t.seq = blockIdx.x / per_seq;
    t.r0 = (blockIdx.x % per_seq) * rows_per_tile;
    t.S = a.seq_lens[t.seq];
    t.ctx = t.S - 1;
    t.token0 = t.seq;
  }
  t.count = min(rows_per_tile, (t.S - t.ctx) * a.H - t.r0);
  return t;
}

template <int NR, int MG>
__global__ __launch_bounds__(256) void latent_attn_kernel(const LatentArgs a) {
  constexpr int RANK = 64 * NR;
  constexpr int ROW = RANK + ROT;
  constexpr int UPR = ROW / 8;             // 16-byte units per row
  constexpr int STEPS = ROW / 32;          // MFMA k-steps of QK^T
  constexpr int TILE_BYTES = KT * ROW * 2;
  constexpr int M = 16 * MG;
  extern __shared__ char lds[];
  bf16_t* const prob = (bf16_t*)(lds + 2 * TILE_BYTES);          // [M][PPAD]
  float* const red = (float*)(prob + M * PPAD);                   // [M][4]
  int* const slots = (int*)(red + M * 4);                         // [2][KT]

  const Tile tl = find_tile(a, M);
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int c = lane & 15, g = lane >> 4;
  const bf16_t* cache = (const bf16_t*)a.cache;
  const int* table = a.tables + (int64_t)tl.seq * a.max_blocks;

  // keys any row of the tile sees
  const int pos_lo = tl.ctx + tl.r0 / a.H;
  const int pos_hi = tl.ctx + (tl.r0 + tl.count - 1) / a.H;
  const int k_begin = max(0, pos_lo - a.window + 1);
  const int k_end = pos_hi + 1;
  const int n_tiles = (k_end - k_begin + KT - 1) / KT;
  const int per_split = (n_tiles + a.n_split - 1) / a.n_split;
  const int t_begin = min(n_tiles, (int)blockIdx.y * per_split);
  const int t_end = min(n_tiles, t_begin + per_split);

  const int64_t row0 = (int64_t)tl.token0 * a.H + tl.r0;
  if (t_begin >= t_end) {  // an empty split; those are a row's last ones
    for (int i = threadIdx.x; i < tl.count; i += 256)
      a.part_ml[(int64_t)blockIdx.y * a.rows + row0 + i] = float2{NEG, -1.f};
    return;
  }

  // B fragments of the queries: lane's row c, 8 consecutive dims per step
  bf16x8_v qf[MG][STEPS];
  int qpos[MG];
#pragma unroll
  for (int m = 0; m < MG; ++m) {
    const int r = m * 16 + c;
    const bool live = r < tl.count;
    qpos[m] = live ? tl.ctx + (tl.r0 + r) / a.H : -1;  // -1 sees no key
    const int64_t row = row0 + (live ? r : 0);
    const bf16_t* qr = (const bf16_t*)a.q + row * RANK + g * 8;
#pragma unroll
    for (int s = 0; s < RANK / 32; ++s) qf[m][s] = *(const bf16x8_v*)(qr + s * 32);
    // the rest is rotated on the way in: 4 pairs a lane and step
    const bf16_t* rr = (const bf16_t*)a.q_rot + row / a.H * a.rot_token +
                       row % a.H * a.rot_head + g * 8;
    const int pairs = a.rot_dim >> 1;
    const float* ct = a.cos_sin + (int64_t)max(qpos[m], 0) * pairs;
    const float* st = ct + a.positions * pairs;
#pragma unroll
    for (int s = 0; s < ROT / 32; ++s) {
      bf16x8_v q8 = *(const bf16x8_v*)(rr + s * 32);
#pragma unroll
      for (int p = 0; p < 4; ++p) {
        const int i = min(s * 16 + g * 4 + p, pairs - 1);  // padding is zero: any angle
        const float x = (float)q8[2 * p], y = (float)q8[2 * p + 1];
        q8[2 * p] = (__bf16)(x * ct[i] - y * st[i]);
        q8[2 * p + 1] = (__bf16)(y * ct[i] + x * st[i]);
      }
      qf[m][RANK / 32 + s] = q8;
    }
  }

  auto find_slots = [&](int t) {
    if (threadIdx.x < KT) {
      const int k = min(k_begin + t * KT + (int)threadIdx.x, k_end - 1);
      slots[(t & 1) * KT + threadIdx.x] = table[k / a.kv_block] * a.kv_block + k % a.kv_block;
    }
  };
  // piece = 1 KiB of the tile image; lane-linear in LDS, swizzled at the source
  auto stage = [&](int t) {
    char* dst = lds + (t & 1) * TILE_BYTES;
#pragma unroll
    for (int i = 0; i < TILE_BYTES / 4096; ++i) {
      const int piece = i * 4 + wid;
      const int u = piece * 64 + lane;
      const int key = u / UPR;
      const int sw = ((key & 3) << 1) | ((key >> 2) & 1);
      const int unit = (u - key * UPR) ^ sw;
      const bf16_t* src = cache + (int64_t)slots[(t & 1) * KT + key] * ROW + unit * 8;
      __builtin_amdgcn_global_load_lds((glob_char*)src, (lds_char*)(dst + piece * 1024),
                                       16, 0, 0);
    }
  };

  find_slots(t_begin);
  if (t_begin + 1 < t_end) find_slots(t_begin + 1);
  __syncthreads();
  stage(t_begin);

  f32x4_v o[MG][NR] = {};
  // a sink is the softmax's starting state: its maximum, one term of the sum, no value
  const bool sink = a.sink && blockIdx.y == 0;
  float m_run[MG], l_run[MG];
#pragma unroll
  for (int m = 0; m < MG; ++m) {
    m_run[m] = sink ? a.sink[(tl.r0 + m * 16 + c) % a.H] * 1.44269504088896f : NEG;
    l_run[m] = sink && wid == 0 && g == 0 ? 1.f : 0.f;
  }
  const float scale2 = a.scale * 1.44269504088896f;  // exp2 domain
  const int sw_c = ((c & 3) << 1) | ((c >> 2) & 1);

  for (int t = t_begin; t < t_end; ++t) {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();  // tile t landed for every wave; tile t-1 is fully read
    if (t + 1 < t_end) stage(t + 1);
    const char* tile = lds + (t & 1) * TILE_BYTES;

    // scores: lane holds query row c, keys wid*16 + 4g + {0..3}
    f32x4_v s[MG] = {};
    {
      const char* krow = tile + (wid * 16 + c) * (ROW * 2);
#pragma unroll
      for (int st = 0; st < STEPS; ++st) {
        const bf16x8_v kf = *(const bf16x8_v*)(krow + (((st * 4 + g) ^ sw_c) << 4));
#pragma unroll
        for (int m = 0; m < MG; ++m)
          s[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[m][st], s[m], 0, 0, 0);
      }
    }
    const int key0 = k_begin + t * KT + wid * 16 + 4 * g;
#pragma unroll
    for (int m = 0; m < MG; ++m) {
      float mt = NEG;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = key0 + r;
        const bool see = key <= qpos[m] && qpos[m] - key < a.window;
        s[m][r] = see ? s[m][r] * scale2 : -INFINITY;
        mt = fmaxf(mt, s[m][r]);
      }
      mt = fmaxf(mt, __shfl_xor(mt, 16, 64));
      mt = fmaxf(mt, __shfl_xor(mt, 32, 64));
      if (g == 0) red[(m * 16 + c) * 4 + wid] = mt;
    }
    __syncthreads();
#pragma unroll
    for (int m = 0; m < MG; ++m) {
      const float4 w4 = *(const float4*)(red + (m * 16 + c) * 4);
      const float m_new = fmaxf(m_run[m], fmaxf(fmaxf(w4.x, w4.y), fmaxf(w4.z, w4.w)));
      const float alpha = __builtin_amdgcn_exp2f(m_run[m] - m_new);
      m_run[m] = m_new;
      float p[4], sum = 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        p[r] = __builtin_amdgcn_exp2f(s[m][r] - m_new);
        sum += p[r];
      }
      l_run[m] = l_run[m] * alpha + sum;
      store_f<4>(prob + (m * 16 + c) * PPAD + wid * 16 + 4 * g, p);
#pragma unroll
      for (int n = 0; n < NR; ++n) o[m][n] *= alpha;
    }
    if (t + 2 < t_end) find_slots(t + 2);  // tile t's slots were consumed by its stage
    __syncthreads();

    // values: A = latent columns (transposed read), B = probabilities
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      bf16x8_v pf[MG];
#pragma unroll
      for (int m = 0; m < MG; ++m)
        pf[m] = *(const bf16x8_v*)(prob + (m * 16 + c) * PPAD + ks * 32 + g * 8);
      const int key = ks * 32 + g * 8 + (c >> 2);  // and key + 4
      const int sw_lo = (key & 3) << 1;             // (key >> 2) & 1 == 0 here
      const char* v0 = tile + key * (ROW * 2) + (c & 1) * 8;
#pragma unroll
      for (int n = 0; n < NR; ++n) {
        const int unit = (wid * NR + n) * 2 + ((c & 3) >> 1);
        const bf16x4_v lo = __builtin_amdgcn_ds_read_tr16_b64_v4bf16(
            (lds_bf16x4*)(v0 + ((unit ^ sw_lo) << 4)));
        const bf16x4_v hi = __builtin_amdgcn_ds_read_tr16_b64_v4bf16(
            (lds_bf16x4*)(v0 + 4 * (ROW * 2) + ((unit ^ (sw_lo | 1)) << 4)));
        const bf16x8_v vf = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
#pragma unroll
        for (int m = 0; m < MG; ++m)
          o[m][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[m], o[m][n], 0, 0, 0);
      }
    }
  }

  // row sums over the lane groups and waves
  __syncthreads();
#pragma unroll
  for (int m = 0; m < MG; ++m) {
    float l = l_run[m];
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (g == 0) red[(m * 16 + c) * 4 + wid] = l;
  }
  __syncthreads();
#pragma unroll
  for (int m = 0; m < MG; ++m) {
    const int r = m * 16 + c;
    if (r >= tl.count) continue;
    const float4 w4 = *(const float4*)(red + r * 4);
    const float l = w4.x + w4.y + w4.z + w4.w;
    const int64_t row = row0 + r;
    const int col0 = wid * (16 * NR) + 4 * g;
    if (a.n_split == 1) {
      const float inv = l > 0.f ? 1.f / l : 0.f;
      bf16_t* dst = (bf16_t*)a.out + row * RANK + col0;
#pragma unroll
      for (int n = 0; n < NR; ++n) {
        const float v[4] = {o[m][n][0] * inv, o[m][n][1] * inv, o[m][n][2] * inv,
                            o[m][n][3] * inv};
        store_f<4>(dst + n * 16, v);
      }
    } else {
      const int64_t at = (int64_t)blockIdx.y * a.rows + row;
      if (wid == 0 && g == 0) a.part_ml[at] = float2{m_run[m], l};
      float* dst = a.part + at * RANK + col0;
#pragma unroll
      for (int n = 0; n < NR; ++n) *(f32x4_v*)(dst + n * 16) = o[m][n];
    }
  }
}

// Merge the splits (at most 64) of one row.
__global__ __launch_bounds__(128) void split_combine_kernel(
    const SplitOut dst, const float* __restrict__ part, const float2* __restrict__ part_ml,
    const int rows, const int rank, const int n_split) {
  __shared__ float weight[64];
  const int row = blockIdx.x, lane = threadIdx.x & 63;
  const float2 ml = lane < n_split ? part_ml[(int64_t)lane * rows + row] : float2{NEG, -1.f};
  const int live = __popcll(__ballot(ml.y >= 0.f));
  const float m = wave_max(ml.x);
  const float w = ml.y > 0.f ? __builtin_amdgcn_exp2f(ml.x - m) : 0.f;
  const float l = wave_sum(w * fmaxf(ml.y, 0.f));
  const int token = row / dst.H, head = row % dst.H;
  const float gate =
      dst.gate ? sigmoid_f(bf2f(((const bf16_t*)dst.gate)[token * dst.gate_stride + head])) : 1.f;
  if (threadIdx.x < 64) weight[lane] = dst.sum ? gate : l > 0.f ? gate * w / l : 0.f;
  bf16_t* out = (bf16_t*)dst.out + token * dst.out_stride + (int64_t)head * rank;
  __syncthreads();
  for (int i = threadIdx.x * 4; i < rank; i += 512) {
    float acc[4] = {};
    const float* src = part + (int64_t)row * rank + i;
#pragma unroll 8
    for (int s = 0; s < live; ++s) {
      float v[4];
      load_f<4>(v, src + (int64_t)s * rows * rank);
#pragma unroll
      for (int k = 0; k < 4; ++k) acc[k] += weight[s] * v[k];
    }
    store_f<4>(out + i, acc);
  }
}

// Plain kernel for fp32 models and latents beyond the MFMA sizes: one workgroup
// per query row, its 4 waves stride over the keys, a lane holds every 64th dim.
template <typename T, int NE>
__global__ __launch_bounds__(256) void latent_attn_plain_kernel(
    const LatentArgs a, const int rank, const int row) {
  const Tile tl = find_tile(a, 1);
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int64_t qrow = (int64_t)tl.token0 * a.H + tl.r0;
  const int pos = tl.ctx + tl.r0 / a.H;
  const int* table = a.tables + (int64_t)tl.seq * a.max_blocks;
  float q[NE], acc[NE] = {};
#pragma unroll
  for (int e = 0; e < NE; ++e) {
    const int d = e * 64 + lane;
    q[e] = 0.f;
    if (d < rank) {
      q[e] = to_f(((const T*)a.q)[qrow * rank + d]) * a.scale;
    } else if (d < rank + a.rot_dim) {
      const int i = (d - rank) >> 1;
      const T* pair = (const T*)a.q_rot + qrow / a.H * a.rot_token +
                      qrow % a.H * a.rot_head + 2 * i;
      const int64_t at = (int64_t)pos * (a.rot_dim >> 1) + i;
      const float co = a.cos_sin[at];
      const float si = a.cos_sin[a.positions * (a.rot_dim >> 1) + at];
      const float u = to_f(pair[0]), v = to_f(pair[1]);
      q[e] = (d & 1 ? v * co + u * si : u * co - v * si) * a.scale;
    }
  }
  const bool sink = a.sink && wid == 0;
  float m = sink ? a.sink[qrow % a.H] : NEG, l = sink ? 1.f : 0.f;
  for (int k = max(0, pos - a.window + 1) + wid; k <= pos; k += 4) {
    const int64_t slot = (int64_t)table[k / a.kv_block] * a.kv_block + k % a.kv_block;
    const T* kr = (const T*)a.cache + slot * row;
    float kv[NE], dot = 0.f;
#pragma unroll
    for (int e = 0; e < NE; ++e) {
      const int d = e * 64 + lane;
      kv[e] = d < row ? to_f(kr[d]) : 0.f;
      dot += q[e] * kv[e];
    }
    dot = wave_sum(dot);
    const float mn = fmaxf(m, dot);
    const float alpha = __expf(m - mn), p = __expf(dot - mn);
    m = mn;
    l = l * alpha + p;
#pragma unroll
    for (int e = 0; e < NE; ++e) acc[e] = acc[e] * alpha + p * kv[e];
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
    w[i] = __expf(ml[i].x - mx);
    sum += w[i] * ml[i].y;
  }
  for (int d = threadIdx.x; d < rank; d += 256) {
    float v = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) v += w[i] * part[i][d];
    ((T*)a.out)[qrow * rank + d] = from_f<T>(v / sum);
  }
}

template <int NR, int MG>
static void launch_mfma(const LatentArgs& a, int tiles, hipStream_t stream) {
  constexpr int M = 16 * MG;
  constexpr int bytes = 2 * KT * (64 * NR + ROT) * 2 + M * PPAD * 2 + M * 16 + 2 * KT * 4;
  static_assert(bytes <= 160 * 1024, "LDS");
  static bool attr_set = false;
  if (!attr_set) {
    (void)hipFuncSetAttribute((const void*)latent_attn_kernel<NR, MG>,
                              hipFuncAttributeMaxDynamicSharedMemorySize, bytes);
    attr_set = true;
  }
  latent_attn_kernel<NR, MG><<<dim3(tiles, a.n_split), 256, bytes, stream>>>(a);
}

template <int NR>
static void launch_mg(const LatentArgs& a, int mg, int tiles, hipStream_t stream) {
  if (mg == 1)
    launch_mfma<NR, 1>(a, tiles, stream);
  else if (mg == 2 || NR > 4)  // query fragments of 64 rows x 448+ dims would spill
    launch_mfma<NR, 2>(a, tiles, stream);
  else if constexpr (NR <= 4)
    launch_mfma<NR, 4>(a, tiles, stream);
}

template <typename T>
static bool launch_plain(const LatentArgs& a, int rank, int row, int tiles,
                         hipStream_t stream) {
  const int ne = (row + 63) / 64;
  if (ne > 32) return false;
  auto k = ne <= 2    ? latent_attn_plain_kernel<T, 2>
           : ne <= 4  ? latent_attn_plain_kernel<T, 4>
           : ne <= 9  ? latent_attn_plain_kernel<T, 9>
           : ne <= 16 ? latent_attn_plain_kernel<T, 16>
                      : latent_attn_plain_kernel<T, 32>;
  k<<<tiles, 256, 0, stream>>>(a, rank, row);
  return true;
}

extern "C" {

void launch_split_combine(const SplitOut* out, const float* part, const float2* part_ml,
                          int rows, int width, int n_split, hipStream_t stream) {
  split_combine_kernel<<<rows, 128, 0, stream>>>(*out, part, part_ml, rows, width, n_split);
}

bool launch_latent_attn(bool bf16, bool mfma, const LatentArgs* a, int rank, int row,
                        int mg, int tiles, hipStream_t stream) {
  if (!mfma)
    return (bf16 ? launch_plain<bf16_t> : launch_plain<float>)(*a, rank, row, tiles, stream);
  switch (rank) {
    case 64: launch_mg<1>(*a, mg, tiles, stream); break;
    case 128: launch_mg<2>(*a, mg, tiles, stream); break;
    case 256: launch_mg<4>(*a, mg, tiles, stream); break;
    case 384: launch_mg<6>(*a, mg, tiles, stream); break;
    case 512: launch_mg<8>(*a, mg, tiles, stream); break;
    default: return false;
  }
  if (a->n_split > 1) {
    const SplitOut out = {a->out, nullptr, (int64_t)a->H * rank, 0, a->H, false};
    launch_split_combine(&out, a->part, a->part_ml, a->rows, rank, a->n_split, stream);
  }
  return true;
}

}  // extern "C"
