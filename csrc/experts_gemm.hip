// The routed experts' products for many rows per expert (gfx950): a grouped GEMM over
// tiles of 256 rows of one expert.
//
// Rows come grouped by expert.  The first product gathers its token rows and applies the
// gated unit to its accumulators: a wave's two 32-column fragments are gate and up of
// the same 32 outputs.  The second reads the grouped rows in place and scatters its
// results to their (token, choice) entries.
//
//   tile 256 rows x 256 weight rows, 8 waves as 2 x 4, wave tile 128 x 64
//   K in chunks of 64, so that a row's part is a whole cache line; two chunks in LDS,
//     loaded straight there as soon as the chunk before the last is read, source
//     address swizzled.  Products go by halves of a chunk: while the first 64 rows of a
//     wave tile multiply, the fragments of the other 64 are read, and while those
//     multiply, the first ones of the next half (raising the priority of multiplying waves
//     made this slower)
//   waves whose last 64 or all 128 rows are beyond the expert's last one skip them
#include "experts.h"
#include "gated_act.h"

typedef __bf16 bf16x8_v __attribute__((ext_vector_type(8)));
typedef float f32x16_v __attribute__((ext_vector_type(16)));
typedef __attribute__((address_space(3))) char lds_char;
typedef __attribute__((address_space(1))) const char glob_char;

#define PANEL 32768  // one operand's chunk: 256 rows of 128 bytes
#define SLOTS 4
#define WAIT_VM(n) asm volatile("s_waitcnt vmcnt(" #n ")" ::: "memory")

template <bool GLU>
__global__ __launch_bounds__(512, 1) void experts_gemm_kernel(const ExpertsArgs a,
                                                              const int tiles_n) {
  extern __shared__ char lds[];
  // workgroups of the tiles in use, a run of them per XCD; bands of 4 row tiles share
  // their weights, neighbouring columns their rows
  const int used = a.offsets[a.E + 1], nwg = used * tiles_n;
  if ((int)blockIdx.x >= nwg) return;
  int tm, tn;
  {
    const int q = nwg >> 3, r = nwg & 7, xcd = blockIdx.x & 7;
    const int id = (xcd < r ? xcd * (q + 1) : r * (q + 1) + (xcd - r) * q) + (blockIdx.x >> 3);
    const int band = id / (4 * tiles_n), rest = id - band * 4 * tiles_n;
    const int high = min(4, used - band * 4);
    tm = band * 4 + rest % high;
    tn = rest / high;
  }
  const int e = a.tile_expert[tm], row0 = a.tile_row[tm];
  const int rows = min(EXPERT_TILE, a.offsets[e + 1] - row0);
  const int o0 = tn * (GLU ? 128 : 256);  // first output

  const int lane = threadIdx.x & 63, wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int wm = wid >> 2, wn = wid & 3;
  const int c = lane & 31, half = lane >> 5;

  // this thread's rows of every panel: 8 threads a row
  const bf16_t *ap[4], *bp[4];
  const bf16_t* w = (const bf16_t*)a.w + (int64_t)e * (GLU ? 2 : 1) * a.O * a.K;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int row = wid * 32 + i * 8 + (lane >> 3);
    const int col = ((lane & 7) ^ (lane >> 3)) * 8;
    const int r = row0 + min(row, rows - 1);
    ap[i] = (const bf16_t*)a.x + (int64_t)(GLU ? a.perm[r] / a.top : r) * a.x_stride + col;
    // 64 weight rows a wave column: 32 gates and the ups beside them, or 64 outputs
    int o = o0 + (GLU ? (row >> 6) * 32 + (row & 31) : row);
    o = min(o, a.O - 1);
    if (GLU && (row & 32)) o += a.O;
    bp[i] = w + (int64_t)o * a.K + col;
  }
  const int chunks = a.K >> 6;
  const int halves = (rows - wm * 128 + 63) >> 6;  // 64-row parts of this wave with rows
  auto stage = [&](int chunk, int buffer) {  // past the end the last one again: not used
    chunk = min(chunk, chunks - 1);
    char* dst = lds + 2 * buffer * PANEL + wid * 4096;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      __builtin_amdgcn_global_load_lds((glob_char*)(ap[i] + chunk * 64),
                                       (lds_char*)(dst + i * 1024), 16, 0, 0);
      __builtin_amdgcn_global_load_lds((glob_char*)(bp[i] + chunk * 64),
                                       (lds_char*)(dst + PANEL + i * 1024), 16, 0, 0);
    }
  };
  // fragments of steps 2q, 2q + 1 (16 of K each), rows 0 and 32 of a panel's part
  const char* la = lds + (wm * 128 + c) * 128;
  const char* lb = lds + PANEL + (wn * 64 + c) * 128;
  int at[4];
#pragma unroll
  for (int s = 0; s < 4; ++s) at[s] = ((s * 2 + half) ^ (c & 7)) * 16;
  auto read = [&](bf16x8_v (&f)[2][2], const char* p, int q) {
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int i = 0; i < 2; ++i) f[i][s] = *(const bf16x8_v*)(p + at[2 * q + s] + i * 4096);
  };
  f32x16_v acc[4][2] = {};
  auto multiply = [&](int h, int s, const bf16x8_v (&af)[2][2], const bf16x8_v (&bf)[2][2]) {
#pragma unroll
    for (int f = 0; f < 2; ++f)
#pragma unroll
      for (int g = 0; g < 2; ++g)
        acc[2 * h + f][g] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(af[f][s], bf[g][s],
                                                                    acc[2 * h + f][g], 0, 0, 0);
  };
  // chunk c is read by every wave, chunk c + 1 has landed for every wave
  auto hand_over = [&](int c) {
    asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
    __builtin_amdgcn_sched_barrier(0);
    stage(c + 2, c & 1);
  };

  stage(0, 0);
  stage(1, 1);
  WAIT_VM(8);
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");

  // both loops pass the same barriers and stage the same chunks
  if (halves >= 2) {
    bf16x8_v a0[2][2], a1[2][2], b[2][2][2];
    read(b[0], lb, 0);
    read(a0, la, 0);
    for (int c0 = 0; c0 < chunks; c0 += 2) {  // K is a multiple of 128
#pragma unroll
      for (int j = 0; j < 4; ++j) {  // half j & 1 of chunk c0 + (j >> 1)
        const int here = (j >> 1) * 2 * PANEL, next = ((j + 1) >> 1 & 1) * 2 * PANEL;
        multiply(0, 0, a0, b[j & 1]);
        __builtin_amdgcn_sched_barrier(0);
        read(a1, la + here + 8192, j & 1);
        __builtin_amdgcn_sched_barrier(0);
        multiply(0, 1, a0, b[j & 1]);
        __builtin_amdgcn_sched_barrier(0);
        if (j & 1) hand_over(c0 + (j >> 1));
        read(b[~j & 1], lb + next, ~j & 1);
        read(a0, la + next, ~j & 1);
        multiply(1, 0, a1, b[j & 1]);
        multiply(1, 1, a1, b[j & 1]);
        __builtin_amdgcn_sched_barrier(0);
      }
    }
  } else {
    for (int c = 0; c < chunks; ++c) {
      if (halves == 1)
#pragma unroll
        for (int q = 0; q < 2; ++q) {
          bf16x8_v a0[2][2], b[2][2];
          const int here = (c & 1) * 2 * PANEL;
          read(b, lb + here, q);
          read(a0, la + here, q);
          multiply(0, 0, a0, b);
          multiply(0, 1, a0, b);
        }
      hand_over(c);
    }
  }
  WAIT_VM(0);  // the loads past the end

  // register r of a fragment: row (r & 3) + 8 (r >> 2) + 4 half, column c
  bf16_t* out = (bf16_t*)a.out;
#pragma unroll
  for (int f = 0; f < 4; ++f)
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int row = wm * 128 + f * 32 + (r & 3) + 8 * (r >> 2) + 4 * half;
      if (row >= rows) continue;
      if (GLU) {
        const int o = o0 + wn * 32 + c;
        if (o >= a.O) continue;
        // through the model's precision, as a GEMM stores it
        const float gate = to_f(from_f<bf16_t>(acc[f][0][r]));
        const float up = to_f(from_f<bf16_t>(acc[f][1][r]));
        out[(int64_t)(row0 + row) * a.O + o] =
            from_f<bf16_t>(clamped_glu_f(gate, up, a.limit, a.alpha, a.offset, a.cubic));
      } else {
        bf16_t* dst = out + (int64_t)a.perm[row0 + row] * a.O;
#pragma unroll
        for (int g = 0; g < 2; ++g) {
          const int o = o0 + wn * 64 + g * 32 + c;
          if (o < a.O) dst[o] = from_f<bf16_t>(acc[f][g][r]);
        }
      }
    }
}

template <bool GLU>
static void launch(const ExpertsArgs& a, hipStream_t stream) {
  static bool attr_set = false;
  if (!attr_set) {
    (void)hipFuncSetAttribute((const void*)experts_gemm_kernel<GLU>,
                              hipFuncAttributeMaxDynamicSharedMemorySize, SLOTS * PANEL);
    attr_set = true;
  }
  const int per = GLU ? 128 : 256;
  const int tiles_n = (a.O + per - 1) / per;
  experts_gemm_kernel<GLU><<<a.tiles * tiles_n, 512, SLOTS * PANEL, stream>>>(a, tiles_n);
}

extern "C" void launch_experts_gemm(bool glu, const ExpertsArgs* a, hipStream_t stream) {
  glu ? launch<true>(*a, stream) : launch<false>(*a, stream);
}
