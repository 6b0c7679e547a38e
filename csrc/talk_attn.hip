// Grouped attention whose heads mix their scores, over the paged cache on the matrix cores
// (gfx950):
//
//   s_h(i, j) = sum_g T[h, g] scale q_g(i) . k_g(j),   softmax over the visible keys
//
// Decode.  The mix moves to the query: s_h is one product of a long query, T's mix of the
// heads that share a key head, side by side for all key heads, with the whole key row.
// A workgroup owns a sequence, or a run of its keys; it builds the long queries in LDS,
// in the order of the matrix cores' fragments.  Its waves take 32 keys at a time, each by
// itself: keys go from memory straight to the matrix cores, weights through a few LDS
// rows to the lanes that hold the values.  The waves meet once, at the end.
//
// Prompts.  There the mix is a product of its own (the long queries would multiply the
// first product by the number of key heads).  A workgroup owns 32 / group tokens with all
// their heads; wave g computes what belongs to key/value head g: raw scores, and values
// times weights.  In between the scores of a tile of 32 keys go through LDS to be mixed,
// a wave per token: 16 keys x heads times heads x heads.  Scores are fp32 and travel as
// three bf16 parts, whose products with a bf16 T lose nothing.
#include "common_t.h"
#include "grouped_attn.h"
#include "latent_attn.h"

typedef __bf16 bf16x8_v __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4_v __attribute__((ext_vector_type(4)));
typedef float f32x4_v __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) char lds_char;
typedef __attribute__((address_space(3))) bf16x4_v lds_bf16x4;

#define NEG -1e30f
#define LOG2E 1.44269504088896f

// what lanes of this wave wrote to LDS is there for its others
DEV void wave_sync() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

// Over the lanes with this lane & 15.  Swapping rows of 16 (halves) of a register with
// itself leaves both members of every pair side by side.
DEV float quad_max(float v) {
  const unsigned b = __float_as_uint(v);
  auto p = __builtin_amdgcn_permlane16_swap(b, b, false, false);
  const unsigned m = __float_as_uint(fmaxf(__uint_as_float(p[0]), __uint_as_float(p[1])));
  p = __builtin_amdgcn_permlane32_swap(m, m, false, false);
  return fmaxf(__uint_as_float(p[0]), __uint_as_float(p[1]));
}
DEV float quad_sum(float v) {
  const unsigned b = __float_as_uint(v);
  auto p = __builtin_amdgcn_permlane16_swap(b, b, false, false);
  const unsigned m = __float_as_uint(__uint_as_float(p[0]) + __uint_as_float(p[1]));
  p = __builtin_amdgcn_permlane32_swap(m, m, false, false);
  return __uint_as_float(p[0]) + __uint_as_float(p[1]);
}

// ------------------------------------------------------------------ decode

#define DEC_ROWS 16  // keys whose weights are in LDS at a time

// HT: 16-head tiles.  A lane holds UL pieces of 8 value dims and the up to GM heads of
// their value head.  grid (sequences, splits).
template <int HT, int GM, int UL>
__global__ __launch_bounds__(256, 2) void talk_decode_kernel(const GroupedArgs a, const int d,
                                                             const int v) {
  extern __shared__ char lds[];
  const int group = a.H / a.G, DK = a.G * d, steps = DK / 32;
  const int units = a.G * v / 8, p_row = a.G * GM + 4;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int c = lane & 15, quad = lane >> 4;
  bf16x8_v* const qf = (bf16x8_v*)lds;                          // [steps][HT][64]
  float* const merged = (float*)lds;                            // [4][H][v], at the end
  const int body = max(steps * HT * 1024, 16 * a.H * v);
  float* const pw = (float*)(lds + body) + wid * (DEC_ROWS + 1) * p_row;
  float* const al = pw + DEC_ROWS * p_row;                      // rescaling
  float2* const ml = (float2*)((float*)(lds + body) + 4 * (DEC_ROWS + 1) * p_row);  // [4][H]

  const int seq = blockIdx.x, pos = a.seq_lens[seq] - 1;
  const int64_t row0 = (int64_t)seq * a.H;
  const int lo = first_key(a, pos), n_keys = pos + 1 - lo;
  // whole blocks of 32 keys per split
  const int blocks = (n_keys + 31) / 32;
  const int per_split = (blocks + a.n_split - 1) / a.n_split * 32;
  const int x0 = lo + min(n_keys, (int)blockIdx.y * per_split);
  const int x1 = min(pos + 1, x0 + per_split);
  if (x0 >= x1) {
    for (int h = threadIdx.x; h < a.H; h += 256)
      a.part_ml[(int64_t)blockIdx.y * a.rows + row0 + h] = float2{NEG, -1.f};
    return;
  }

  {  // long queries, as fragments: step u / 4, lane (u % 4) * 16 + h % 16
    const bf16_t* q = (const bf16_t*)a.q + seq * a.q_stride;
    // a thread has one unit of 8 dims at a time, for every ``turns``-th head
    const int row_units = DK / 8, turns = max(1, 256 / row_units);
    const int turn = row_units < 256 ? threadIdx.x / row_units : 0;
    for (int u = threadIdx.x - turn * row_units; u < row_units && turn < turns; u += 256) {
      const int g0 = u * 8 / d * group, e0 = u * 8 % d;
      float y[GM][8];
#pragma unroll
      for (int g = 0; g < GM; ++g)
        load_f<8>(y[g], q + (int64_t)(g0 + min(g, group - 1)) * d + e0);
#pragma unroll 4
      for (int h = turn; h < 16 * HT; h += turns) {
        float x[8] = {};
#pragma unroll
        for (int g = 0; g < GM; ++g) {
          const float t = a.talk[min(h, a.H - 1) * a.H + g0 + min(g, group - 1)];
          const float f = h < a.H && g < group ? t : 0.f;
#pragma unroll
          for (int e = 0; e < 8; ++e) x[e] += f * y[g][e];
        }
        bf16x8_v f;
#pragma unroll
        for (int e = 0; e < 8; ++e) f[e] = (__bf16)x[e];
        qf[((u >> 2) * HT + (h >> 4)) * 64 + (u & 3) * 16 + (h & 15)] = f;
      }
    }
  }
  __syncthreads();

  const int* table = a.tables + (int64_t)seq * a.max_blocks;
  const bf16_t* kc = (const bf16_t*)a.k_cache + quad * 8;
  const bf16_t* vc = (const bf16_t*)a.v_cache;
  const float mul = a.scale * LOG2E;
  int unit[UL], kvh[UL];
#pragma unroll
  for (int j = 0; j < UL; ++j) {
    unit[j] = min(lane + 64 * j, units - 1);
    kvh[j] = unit[j] * 8 / v;
  }
  int at[HT];  // where this lane's heads are in a row of weights
#pragma unroll
  for (int t = 0; t < HT; ++t) {
    const int h = t * 16 + c;
    at[t] = h / group * GM + h % group;
  }
  float m[HT], l[HT], acc[GM][UL][8];
#pragma unroll
  for (int t = 0; t < HT; ++t) m[t] = NEG, l[t] = 0.f;
#pragma unroll
  for (int g = 0; g < GM; ++g)
#pragma unroll
    for (int j = 0; j < UL; ++j)
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[g][j][e] = 0.f;

  for (int x = x0 + wid * 32; x < x1; x += 128) {
    const int k = min(x + (lane & 31), x1 - 1);
    const int slot = table[k / a.kv_block] * a.kv_block + k % a.kv_block;
    const bf16_t* k0 = kc + (int64_t)__shfl(slot, c, 64) * DK;
    const bf16_t* k1 = kc + (int64_t)__shfl(slot, c + 16, 64) * DK;
    f32x4_v s[2][HT] = {};
#pragma unroll 8
    for (int st = 0; st < steps; ++st) {
      const bf16x8_v f0 = *(const bf16x8_v*)(k0 + st * 32);
      const bf16x8_v f1 = *(const bf16x8_v*)(k1 + st * 32);
#pragma unroll
      for (int t = 0; t < HT; ++t) {
        const bf16x8_v b = qf[(st * HT + t) * 64 + lane];
        s[0][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f0, b, s[0][t], 0, 0, 0);
        s[1][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f1, b, s[1][t], 0, 0, 0);
      }
    }
    // head c + 16 t, keys x + 16 b + 4 quad + r
    float alpha[HT];
    bool moved = false;
#pragma unroll
    for (int t = 0; t < HT; ++t) {
      float mt = m[t];
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          s[b][t][r] = x + 16 * b + 4 * quad + r < x1 ? s[b][t][r] * mul : -INFINITY;
          mt = fmaxf(mt, s[b][t][r]);
        }
      mt = quad_max(mt);
      alpha[t] = __builtin_amdgcn_exp2f(m[t] - mt);
      moved |= mt > m[t];
      m[t] = mt;
      l[t] *= alpha[t];
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          s[b][t][r] = __builtin_amdgcn_exp2f(s[b][t][r] - mt);
          l[t] += s[b][t][r];
        }
    }
    moved = __any(moved);
    const int n = min(32, x1 - x);
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      if (16 * b >= n) break;
      wave_sync();
#pragma unroll
      for (int t = 0; t < HT; ++t)
        if (t * 16 + c < a.H) {
#pragma unroll
          for (int r = 0; r < 4; ++r) pw[(4 * quad + r) * p_row + at[t]] = s[b][t][r];
          if (b == 0 && quad == 0) al[at[t]] = alpha[t];
        }
      wave_sync();
      if (b == 0 && moved) {
#pragma unroll
        for (int j = 0; j < UL; ++j)
#pragma unroll
          for (int g = 0; g < GM; ++g) {
            const float f = al[kvh[j] * GM + g];
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[g][j][e] *= f;
          }
      }
      constexpr int AHEAD = UL <= 2 ? 8 : 4;
#pragma unroll
      for (int i0 = 0; i0 < 16; i0 += AHEAD) {
        Pack<bf16_t, 8> val[AHEAD][UL];
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) {  // past the end: the last key again, weight 0
          const int64_t sl = __builtin_amdgcn_readlane(slot, 16 * b + i0 + i);
#pragma unroll
          for (int j = 0; j < UL; ++j)
            val[i][j] = *(const Pack<bf16_t, 8>*)(vc + (sl * units + unit[j]) * 8);
        }
#pragma unroll
        for (int i = 0; i < AHEAD; ++i)
#pragma unroll
          for (int j = 0; j < UL; ++j) {
            const Pack<float, GM> p = *(const Pack<float, GM>*)(pw + (i0 + i) * p_row + kvh[j] * GM);
#pragma unroll
            for (int e = 0; e < 8; ++e) {
              const float y = to_f(val[i][j].v[e]);
#pragma unroll
              for (int g = 0; g < GM; ++g) acc[g][j][e] += p.v[g] * y;
            }
          }
      }
    }
  }

  __syncthreads();  // the long queries are read
#pragma unroll
  for (int t = 0; t < HT; ++t) {
    const float sum = quad_sum(l[t]);
    if (quad == 0 && t * 16 + c < a.H) ml[wid * a.H + t * 16 + c] = float2{m[t], sum};
  }
#pragma unroll
  for (int j = 0; j < UL; ++j) {
    if (lane + 64 * j >= units) continue;
    const int e0 = unit[j] * 8 % v;
#pragma unroll
    for (int g = 0; g < GM; ++g)
      if (g < group) {
        float* o = merged + ((int64_t)wid * a.H + kvh[j] * group + g) * v + e0;
        *(f32x4_v*)o = f32x4_v{acc[g][j][0], acc[g][j][1], acc[g][j][2], acc[g][j][3]};
        *(f32x4_v*)(o + 4) = f32x4_v{acc[g][j][4], acc[g][j][5], acc[g][j][6], acc[g][j][7]};
      }
  }
  __syncthreads();
  for (int i = threadIdx.x; i < a.H * v; i += 256) {
    const int h = i / v, e = i - h * v;
    float mx = NEG, sum = 0.f, o = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) mx = fmaxf(mx, ml[w * a.H + h].x);
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float f = __builtin_amdgcn_exp2f(ml[w * a.H + h].x - mx);
      sum += f * ml[w * a.H + h].y;
      o += f * merged[(int64_t)w * a.H * v + i];
    }
    if (a.n_split == 1) {
      ((bf16_t*)a.out)[seq * a.out_stride + i] = from_f<bf16_t>(o / sum);
    } else {
      const int64_t r = (int64_t)blockIdx.y * a.rows + row0 + h;
      a.part[r * v + e] = o;
      if (e == 0) a.part_ml[r] = float2{mx, sum};
    }
  }
}

static int decode_bytes(const GroupedArgs& a, int d, int v, int ht, int gm) {
  const int q = a.G * d / 32 * ht * 1024, o = 16 * a.H * v;
  return (q > o ? q : o) + 16 * (DEC_ROWS + 1) * (a.G * gm + 4) + 32 * a.H;
}

template <int HT, int GM, int UL>
static void launch_decode(const GroupedArgs& a, int d, int v, int seqs, hipStream_t stream) {
  static bool attr_set = false;
  if (!attr_set) {
    (void)hipFuncSetAttribute((const void*)talk_decode_kernel<HT, GM, UL>,
                              hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    attr_set = true;
  }
  talk_decode_kernel<HT, GM, UL>
      <<<dim3(seqs, a.n_split), 256, decode_bytes(a, d, v, HT, GM), stream>>>(a, d, v);
}

template <int HT, int GM>
static void launch_decode_units(const GroupedArgs& a, int d, int v, int seqs,
                                hipStream_t stream) {
  const int ul = (a.G * v / 8 + 63) / 64;
  if (ul <= 1)
    launch_decode<HT, GM, 1>(a, d, v, seqs, stream);
  else if (ul <= 2)
    launch_decode<HT, GM, 2>(a, d, v, seqs, stream);
  else if constexpr (GM <= 4)
    launch_decode<HT, GM, 4>(a, d, v, seqs, stream);
}

template <int HT>
static void launch_decode_group(const GroupedArgs& a, int d, int v, int gm, int seqs,
                                hipStream_t stream) {
  (gm == 1   ? launch_decode_units<HT, 1>
   : gm == 2 ? launch_decode_units<HT, 2>
   : gm == 4 ? launch_decode_units<HT, 4>
             : launch_decode_units<HT, 8>)(a, d, v, seqs, stream);
}

// ------------------------------------------------------------------ prompts

#define KT 32   // keys of a tile
#define PARTS 3  // bf16 parts of a score

// Eight scores as fragments of the mix: top, middle and low 8 bits of their 24.
DEV void split_scores(const float* x, bf16x8_v* part) {
  unsigned w[PARTS][4];
#pragma unroll
  for (int e = 0; e < 8; e += 2) {
    float lo = x[e], hi = x[e + 1];
#pragma unroll
    for (int n = 0; n < PARTS; ++n) {
      const unsigned l = __float_as_uint(lo), h = __float_as_uint(hi);
      w[n][e / 2] = __builtin_amdgcn_perm(h, l, 0x07060302);  // upper halves
      lo -= __uint_as_float(l & 0xffff0000u);
      hi -= __uint_as_float(h & 0xffff0000u);
    }
  }
#pragma unroll
  for (int n = 0; n < PARTS; ++n) part[n] = __builtin_bit_cast(bf16x8_v, w[n]);
}

// 16 bytes a lane, from src (the same in all lanes) + offset straight to LDS, lanes side by
// side.  As assembly, since the compiler would wait for the builtin's loads ahead of every
// LDS access; the caller waits, once.
DEV void load_to_lds(unsigned dst, const char* src, unsigned offset) {
  const uint64_t p = (uint64_t)src;
  const uint64_t at = (uint64_t)__builtin_amdgcn_readfirstlane((unsigned)(p >> 32)) << 32 |
                      (unsigned)__builtin_amdgcn_readfirstlane((unsigned)p);
  asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, %2"
               :: "s"(dst), "v"(offset), "s"(at) : "memory", "m0");
}

// unit of a key's values in LDS: the keys that one transposing read takes are spread over
// the banks
template <int VU>
DEV int swizzled(int unit, int key) {
  return unit ^ (((key & 3) << 1 | (key >> 2 & 1) | (key & 8)) & (VU - 1));
}

struct PromptLds {  // offsets in bytes
  int pitch, weights, values, alpha, stats, lows, total;
};

// weights of one key/value head: 32 rows of KT bf16, and an offset between heads that
// spreads them over the banks
#define W_HEAD (32 * KT * 2 + 32)

static __host__ __device__ inline PromptLds prompt_lds(int H, int G, int tokens, int v) {
  PromptLds l;
  // of a (token, key) pair's fp32 scores, an odd number of 16-byte units
  l.pitch = ((H + 3) / 4 | 1) * 16;
  l.weights = tokens * KT * l.pitch;            // [2][G] W_HEAD
  l.values = l.weights + 2 * G * W_HEAD;        // [G][KT][v] bf16, swizzled
  l.alpha = l.values + G * KT * v * 2;          // [2][G][32]
  l.stats = l.alpha + 2 * G * 32 * 4;           // [tokens][H] maximum and sum
  l.lows = l.stats + tokens * H * 8;            // [tokens] first visible key
  l.total = l.lows + tokens * 4;
  return l;
}

// G waves, wave g for key/value head g: 32 rows, token * group + head of the group.
// HT: 16-head tiles of the mix, KH: its inner steps of 32 heads.  GV: heads of a group that
// are stored together, 4, 2 or 1.
//
// Between two barriers a wave mixes a tile's scores for its tokens, makes the next tile's
// raw scores and adds the last tile's values; the raw scores then replace the mixed ones.
template <int DN, int VN, int HT, int GV>
__global__ __launch_bounds__(512, 2) void talk_prefill_kernel(const GroupedArgs a) {
  constexpr int D = 64 * DN, V = 64 * VN, STEPS = D / 32, VT = V / 16, VU = V / 8;
  constexpr int KH = (HT + 1) / 2;
  extern __shared__ char lds[];
  const int group = a.H / a.G, TQ = 32 / group;
  const PromptLds L = prompt_lds(a.H, a.G, TQ, V);
  const int tile = a.n_tiles - 1 - blockIdx.x;
  const int seq = a.tile_seq[tile], q0 = a.tile_q0[tile];
  const int ctx = a.ctx_lens[seq];
  const int tokens = min(TQ, a.seq_lens[seq] - ctx - q0);
  const int64_t row0 = a.row_starts[seq] + q0;
  const int* table = a.tables + (int64_t)seq * a.max_blocks;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int c = lane & 15, quad = lane >> 4;

  // scores beyond the heads stay zero
  for (int i = threadIdx.x; i < L.weights / 16; i += blockDim.x)
    ((ulonglong2*)lds)[i] = ulonglong2{0, 0};
  float2* const stats = (float2*)(lds + L.stats);
  for (int i = threadIdx.x; i < TQ * a.H; i += blockDim.x) stats[i] = float2{NEG, 0.f};
  int* const lows = (int*)(lds + L.lows);
  if ((int)threadIdx.x < tokens) lows[threadIdx.x] = first_key(a, ctx + q0 + threadIdx.x);

  // this wave's queries; row 16 i + c.  Rows past the end repeat valid ones
  bf16x8_v qf[2][STEPS];
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int r = 16 * i + c, t = min(r / group, tokens - 1);
    const bf16_t* q = (const bf16_t*)a.q + (row0 + t) * a.q_stride +
                      (int64_t)(wid * group + r % group) * D + quad * 8;
#pragma unroll
    for (int s = 0; s < STEPS; ++s) qf[i][s] = *(const bf16x8_v*)(q + s * 32);
  }
  // T, as the fragments of its product: output head 16 t + c, input heads 32 k + 8 quad ..
  bf16x8_v tf[HT][KH];
#pragma unroll
  for (int t = 0; t < HT; ++t)
#pragma unroll
    for (int k = 0; k < KH; ++k) {
      float x[8];
#pragma unroll
      for (int e = 0; e < 8; ++e)
        x[e] = a.talk[min(16 * t + c, a.H - 1) * a.H + min(32 * k + 8 * quad + e, a.H - 1)];
#pragma unroll
      for (int e = 0; e < 8; ++e)
        tf[t][k][e] = (__bf16)(16 * t + c < a.H && 32 * k + 8 * quad + e < a.H ? x[e] : 0.f);
    }

  const int k_end = ctx + q0 + tokens;
  const int first = first_key(a, ctx + q0) / KT * KT;
  const int n_tiles = (k_end - first + KT - 1) / KT;
  const int k_row = a.G * D * 2, v_row = a.G * V * 2;  // bytes of a cached key and value
  const int me = __builtin_amdgcn_readfirstlane(wid);
  const char* const kc = (const char*)a.k_cache + me * D * 2;
  const char* const vc = (const char*)a.v_cache + me * V * 2;
  char* const values = lds + L.values + wid * KT * V * 2;
  // 16 keys lie in one page: everything about them but a lane's constant offset is scalar
  struct Half {
    int page, in;  // place in the table, first key within the page
  };
  Half ahead = {first / a.kv_block, first % a.kv_block};
  const int last_page = (k_end - 1) / a.kv_block;
  int blocks[2], ins[2];  // of the tile after those whose slots are known
  auto look_up = [&]() {
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      blocks[b] = table[min(ahead.page, last_page)];
      ins[b] = ahead.in;
      ahead.in += 16;
      if (ahead.in == a.kv_block) ahead = {ahead.page + 1, 0};
    }
  };
  struct Slots {
    int64_t of[2];
  };
  auto found = [&]() {
    Slots s;
#pragma unroll
    for (int b = 0; b < 2; ++b)
      s.of[b] = (int64_t)__builtin_amdgcn_readfirstlane(blocks[b]) * a.kv_block + ins[b];
    return s;
  };
  bf16x8_v kf[2][STEPS];
  const unsigned k_lane = c * k_row + quad * 16;
  auto load_keys = [&](const Slots& s) {
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      const char* k = kc + s.of[b] * k_row;
#pragma unroll
      for (int st = 0; st < STEPS; ++st)
        kf[b][st] = *(const bf16x8_v*)(k + (k_lane + st * 64));
    }
  };
  constexpr int KEYS = 64 / VU;  // of a load; a lane's place in one repeats every 16 keys
  unsigned v_lane[16 / KEYS];
#pragma unroll
  for (int i = 0; i < 16 / KEYS; ++i) {
    const int key = i * KEYS + lane / VU;
    v_lane[i] = key * v_row + swizzled<VU>(lane % VU, key) * 16;
  }
  const unsigned v_dst =
      __builtin_amdgcn_readfirstlane((unsigned)(uintptr_t)(lds_char*)values);
  auto load_values = [&](const Slots& s) {  // for this wave alone
#pragma unroll
    for (int i = 0; i < KT / KEYS; ++i)
      load_to_lds(v_dst + i * 1024, vc + s.of[i * KEYS / 16] * v_row, v_lane[i % (16 / KEYS)]);
  };
  // keys past the end have weight zero, but what lies there need not be a number
  auto clear_values = [&](int from) {
    for (int i = from * VU + lane; i < KT * VU; i += 64)
      ((ulonglong2*)values)[i] = ulonglong2{0, 0};
  };

  const float mul = a.scale * LOG2E;
  // where this lane's rows 16 i + 4 quad + (0, GV, ..) of raw scores go, or -1
  int put[2][4 / GV];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int r = 0; r < 4 / GV; ++r) {
      const int row = 16 * i + 4 * quad + r * GV;
      put[i][r] = row < TQ * group ? (row / group * KT + c) * L.pitch +
                                         (wid * group + row % group) * 4 : -1;
    }
  f32x4_v raw[2][2];  // key 16 b + c, rows 16 i + 4 quad + r
  auto score = [&]() {
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int i = 0; i < 2; ++i) raw[b][i] = f32x4_v{};
#pragma unroll
    for (int st = 0; st < STEPS; ++st)
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int i = 0; i < 2; ++i)
          raw[b][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[i][st], kf[b][st], raw[b][i], 0,
                                                              0, 0);
  };
  auto put_scores = [&]() {
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const f32x4_v s = raw[b][i] * mul;
#pragma unroll
        for (int r = 0; r < 4 / GV; ++r) {
          if (put[i][r] < 0) continue;
          float* at = (float*)(lds + put[i][r] + 16 * b * L.pitch);
          if constexpr (GV == 4) {
            *(f32x4_v*)at = s;
          } else {
#pragma unroll
            for (int e = 0; e < GV; ++e) at[e] = s[r * GV + e];
          }
        }
      }
  };
  f32x4_v o[2][VT] = {};  // rows 16 i + 4 quad + r, dims 16 n + c
  auto add_values = [&](int t) {
    const char* weights = lds + L.weights + ((t & 1) * a.G + wid) * W_HEAD;
    const float* alpha = (const float*)(lds + L.alpha) + ((t & 1) * a.G + wid) * 32;
    f32x4_v f[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) f[i] = *(const f32x4_v*)(alpha + 16 * i + 4 * quad);
    bool moved = false;
#pragma unroll
    for (int r = 0; r < 4; ++r) moved |= f[0][r] != 1.f || f[1][r] != 1.f;
    if (__any(moved)) {
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int n = 0; n < VT; ++n) o[i][n] *= f[i];
    }
    bf16x8_v pf[2];
#pragma unroll
    for (int i = 0; i < 2; ++i)
      pf[i] = *(const bf16x8_v*)(weights + (16 * i + c) * KT * 2 + quad * 16);
    const int key = quad * 8 + (c >> 2);
    const char* vrow = values + key * V * 2 + (c & 1) * 8;
#pragma unroll
    for (int n = 0; n < VT; ++n) {
      const int unit = n * 2 + ((c & 3) >> 1);
      const bf16x4_v a0 = __builtin_amdgcn_ds_read_tr16_b64_v4bf16(
          (lds_bf16x4*)(vrow + (swizzled<VU>(unit, key) << 4)));
      const bf16x4_v a1 = __builtin_amdgcn_ds_read_tr16_b64_v4bf16(
          (lds_bf16x4*)(vrow + 4 * V * 2 + (swizzled<VU>(unit, key + 4) << 4)));
      const bf16x8_v vf = __builtin_shufflevector(a0, a1, 0, 1, 2, 3, 4, 5, 6, 7);
#pragma unroll
      for (int i = 0; i < 2; ++i)
        o[i][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf[i], vf, o[i][n], 0, 0, 0);
    }
  };

  // slots of tiles t and t + 1, pages of tile t + 2
  look_up();
  Slots here = found();
  load_keys(here);
  look_up();
  Slots next = found();
  look_up();
  __syncthreads();
  score();
  load_keys(next);
  put_scores();
  __syncthreads();

  for (int t = 0; t < n_tiles; ++t) {
    const int key0 = first + t * KT;
    // a wave per token: head 16 h + c, keys key0 + 16 b + 4 quad + r
    for (int q = wid; q < tokens; q += a.G) {
      const int pos = ctx + q0 + q, lo = lows[q];
      f32x4_v s[2][HT] = {};
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        const char* src = lds + (q * KT + 16 * b + c) * L.pitch;
#pragma unroll
        for (int k = 0; k < KH; ++k) {
          float x[8];
#pragma unroll
          for (int e = 0; e < 8; e += 4) {
            const int at = (32 * k + 8 * quad + e) * 4;
            f32x4_v y = {};
            if (at < L.pitch) y = *(const f32x4_v*)(src + at);
#pragma unroll
            for (int i = 0; i < 4; ++i) x[e + i] = y[i];
          }
          bf16x8_v f[PARTS];
          split_scores(x, f);
#pragma unroll
          for (int n = 0; n < PARTS; ++n)
#pragma unroll
            for (int h = 0; h < HT; ++h)
              s[b][h] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f[n], tf[h][k], s[b][h], 0, 0, 0);
        }
      }
      if (key0 + KT - 1 > pos || key0 < lo) {
#pragma unroll
        for (int b = 0; b < 2; ++b)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int key = key0 + 16 * b + 4 * quad + r;
            const bool seen = key <= pos && key >= lo;
#pragma unroll
            for (int h = 0; h < HT; ++h) s[b][h][r] = seen ? s[b][h][r] : -INFINITY;
          }
      }
#pragma unroll
      for (int n = 0; n < HT; ++n) {
        const int h = 16 * n + c;
        const bool has = h < a.H;
        float mt = NEG;
#pragma unroll
        for (int b = 0; b < 2; ++b)
#pragma unroll
          for (int r = 0; r < 4; ++r) mt = fmaxf(mt, s[b][n][r]);
        const float2 old = stats[q * a.H + (has ? h : 0)];
        mt = fmaxf(quad_max(mt), old.x);
        float sum = 0.f;
        const int g = (t & 1) * a.G + h / group, row = q * group + h % group;
        char* dst = lds + L.weights + g * W_HEAD + row * KT * 2 + quad * 8;
#pragma unroll
        for (int b = 0; b < 2; ++b) {
          float p[4];
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            p[r] = __builtin_amdgcn_exp2f(s[b][n][r] - mt);
            sum += p[r];
          }
          if (has) store_f<4>((bf16_t*)(dst + b * 32), p);
        }
        sum = quad_sum(sum);
        if (has && quad == 0) {
          const float f = __builtin_amdgcn_exp2f(old.x - mt);
          stats[q * a.H + h] = float2{mt, old.y * f + sum};
          ((float*)(lds + L.alpha))[g * 32 + row] = f;
        }
      }
    }
    score();  // of tile t + 1
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");      // the last tile's values are here
    const Slots after = found();
    load_keys(after);
    if (t > 0) {
      add_values(t - 1);
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // and may be overwritten
    }
    load_values(here);
    here = next;
    next = after;
    look_up();
    __syncthreads();
    put_scores();
    __syncthreads();
  }
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  clear_values(k_end - (first + (n_tiles - 1) * KT));
  wave_sync();
  add_values(n_tiles - 1);

#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = 16 * i + 4 * quad + r, t = row / group;
      if (t >= tokens || t >= TQ) continue;
      const int h = wid * group + row % group;
      const float inv = 1.f / stats[t * a.H + h].y;
      bf16_t* dst = (bf16_t*)a.out + (row0 + t) * a.out_stride + (int64_t)h * V + c;
#pragma unroll
      for (int n = 0; n < VT; ++n) dst[16 * n] = from_f<bf16_t>(o[i][n][r] * inv);
    }
}

template <int DN, int VN, int HT, int GV>
static bool launch_prefill(const GroupedArgs& a, hipStream_t stream) {
  const int bytes = prompt_lds(a.H, a.G, 32 / (a.H / a.G), 64 * VN).total;
  if (bytes > 160 * 1024) return false;
  static bool attr_set = false;
  if (!attr_set) {
    (void)hipFuncSetAttribute((const void*)talk_prefill_kernel<DN, VN, HT, GV>,
                              hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    attr_set = true;
  }
  talk_prefill_kernel<DN, VN, HT, GV><<<a.n_tiles, 64 * a.G, bytes, stream>>>(a);
  return true;
}

template <int DN, int VN, int HT>
static bool launch_prefill_group(const GroupedArgs& a, hipStream_t stream) {
  const int group = a.H / a.G;
  return group % 4 == 0   ? launch_prefill<DN, VN, HT, 4>(a, stream)
         : group % 2 == 0 ? launch_prefill<DN, VN, HT, 2>(a, stream)
                          : launch_prefill<DN, VN, HT, 1>(a, stream);
}

template <int DN, int VN>
static bool launch_prefill_heads(const GroupedArgs& a, hipStream_t stream) {
  return a.H <= 16   ? launch_prefill_group<DN, VN, 1>(a, stream)
         : a.H <= 32 ? launch_prefill_group<DN, VN, 2>(a, stream)
                     : launch_prefill_group<DN, VN, 4>(a, stream);
}

static bool mixes(const GroupedArgs& a) {
  return a.talk && !a.sink && !a.bias && !a.gate && !a.sigmoid && a.cap == 0.f && a.keep == 0;
}

extern "C" {

// Tokens per workgroup of the prompt kernel for these sizes; 0: the plain kernel.
int talk_prefill_tokens(int H, int G, int d, int v, int kv_block) {
  if (kv_block % 16) return 0;
  const int group = H / G;
  if ((d != 64 && d != 128) || (v != 64 && v != 128) || G > 8 || H > 64 || group > 32) return 0;
  return prompt_lds(H, G, 32 / group, v).total <= 160 * 1024 ? 32 / group : 0;
}

bool launch_talk_prefill(const GroupedArgs* a, int d, int v, hipStream_t stream) {
  if (!mixes(*a) || !talk_prefill_tokens(a->H, a->G, d, v, a->kv_block)) return false;
  if (d == 64)
    return v == 64 ? launch_prefill_heads<1, 1>(*a, stream) : launch_prefill_heads<1, 2>(*a, stream);
  return v == 64 ? launch_prefill_heads<2, 1>(*a, stream) : launch_prefill_heads<2, 2>(*a, stream);
}

static int group_width(int group) { return group <= 1 ? 1 : group <= 2 ? 2 : group <= 4 ? 4 : 8; }

// Does the decode kernel take these sizes?
bool talk_decode_fits(int H, int G, int d, int v) {
  GroupedArgs a{};
  a.H = H;
  a.G = G;
  const int gm = group_width(H / G), ul = (G * v / 8 + 63) / 64;
  return d % 64 == 0 && v % 64 == 0 && H <= 64 && H / G <= 8 && ul <= (gm == 8 ? 2 : 4) &&
         decode_bytes(a, d, v, H <= 16 ? 1 : H <= 32 ? 2 : 4, gm) <= 160 * 1024;
}

bool launch_talk_decode(const GroupedArgs* a, int d, int v, int seqs, hipStream_t stream) {
  if (!mixes(*a) || !talk_decode_fits(a->H, a->G, d, v)) return false;
  const int gm = group_width(a->H / a->G);
  (a->H <= 16   ? launch_decode_group<1>
   : a->H <= 32 ? launch_decode_group<2>
                : launch_decode_group<4>)(*a, d, v, gm, seqs, stream);
  if (a->n_split > 1) {
    const SplitOut out = {a->out, a->gate, a->out_stride, a->gate_stride, a->H, a->sigmoid};
    launch_split_combine(&out, a->part, a->part_ml, a->rows, v, a->n_split, stream);
  }
  return true;
}

}  // extern "C"
