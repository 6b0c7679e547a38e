// The routed experts' products for many rows per expert (gfx950): a grouped GEMM over
// tiles of 256 rows of one expert, on the schedule of gemm_bf16.hip.
//
// Rows come grouped by expert.  The first product gathers its token rows and applies the
// gated unit to its accumulators: a wave's two 32-column fragments are gate and up of
// the same 32 outputs.  The second reads the grouped rows in place and scatters its
// results to their (token, choice) entries.
//
//   tile 256 rows x 256 weight rows, 8 waves as 2 x 4, wave tile 128 x 64
//   K in chunks of 32: LDS ring of 8 panels of 16 KiB, a panel is one chunk of either
//     operand, loaded straight to LDS 6 phases ahead of its use, source address swizzled
//   phase = (chunk, half of the rows); loads are counted, never drained in the loop
#include "experts.h"
#include "gated_act.h"

typedef __bf16 bf16x8_v __attribute__((ext_vector_type(8)));
typedef float f32x16_v __attribute__((ext_vector_type(16)));
typedef __attribute__((address_space(3))) char lds_char;
typedef __attribute__((address_space(1))) const char glob_char;

#define PANEL 16384
#define SLOTS 8
#define WAIT_VM(n) asm volatile("s_waitcnt vmcnt(" #n ")" ::: "memory")
#define WAIT_LGKM0() asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory")

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

  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int wm = wid >> 2, wn = wid & 3;
  const int c = lane & 31, half = lane >> 5;

  // this thread's two rows of every panel
  const bf16_t *ap[2], *bp[2];
  const bf16_t* w = (const bf16_t*)a.w + (int64_t)e * (GLU ? 2 : 1) * a.O * a.K;
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int row = wid * 32 + i * 16 + (lane >> 2);
    const int col = ((lane & 3) ^ ((row >> 2) & 3)) * 8;
    const int r = row0 + min(row, rows - 1);
    ap[i] = (const bf16_t*)a.x + (int64_t)(GLU ? a.perm[r] / a.top : r) * a.x_stride + col;
    // 64 weight rows a wave column: 32 gates and the ups beside them, or 64 outputs
    int o = o0 + (GLU ? (row >> 6) * 32 + (row & 31) : row);
    o = min(o, a.O - 1);
    if (GLU && (row & 32)) o += a.O;
    bp[i] = w + (int64_t)o * a.K + col;
  }
  auto stage = [&](const bf16_t* const* p, int chunk, int slot) {
#pragma unroll
    for (int i = 0; i < 2; ++i)
      __builtin_amdgcn_global_load_lds((glob_char*)(p[i] + chunk * 32),
                                       (lds_char*)(lds + slot * PANEL + wid * 2048 + i * 1024),
                                       16, 0, 0);
  };

  const int ra = wm * 128 + c, rb = wn * 64 + c;
  int off_a[2], off_b[2];
#pragma unroll
  for (int s = 0; s < 2; ++s) {
    off_a[s] = ra * 64 + (((s << 1) | half) ^ ((ra >> 2) & 3)) * 16;
    off_b[s] = rb * 64 + (((s << 1) | half) ^ ((rb >> 2) & 3)) * 16;
  }
  const int chunks = a.K >> 5, phases = chunks << 1;  // K is a multiple of 128

#pragma unroll
  for (int p = 0; p < 6; ++p) stage(p & 1 ? bp : ap, p >> 1, p);
  WAIT_VM(8);
  __builtin_amdgcn_s_barrier();

  f32x16_v acc[4][2] = {};
  for (int ph0 = 0; ph0 < phases; ph0 += 8) {
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int h = j & 1;
      const char* pa = lds + (2 * (j >> 1)) * PANEL;
      const char* pb = pa + PANEL;
      bf16x8_v af[2][2], bf[2][2];
#pragma unroll
      for (int s = 0; s < 2; ++s)
#pragma unroll
        for (int f = 0; f < 2; ++f) {
          af[f][s] = *(const bf16x8_v*)(pa + off_a[s] + (2 * h + f) * 2048);
          bf[f][s] = *(const bf16x8_v*)(pb + off_b[s] + f * 2048);
        }
      // past the end the last chunk again, into slots that nobody reads
      stage(j & 1 ? bp : ap, min((ph0 + j + 6) >> 1, chunks - 1), (j + 6) & 7);
      __builtin_amdgcn_s_barrier();
      WAIT_LGKM0();
      __builtin_amdgcn_s_setprio(1);
#pragma unroll
      for (int s = 0; s < 2; ++s)
#pragma unroll
        for (int f = 0; f < 2; ++f)
#pragma unroll
          for (int g = 0; g < 2; ++g)
            acc[2 * h + f][g] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
                af[f][s], bf[g][s], acc[2 * h + f][g], 0, 0, 0);
      __builtin_amdgcn_s_setprio(0);
      if (h) WAIT_VM(8);
      __builtin_amdgcn_s_barrier();
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
