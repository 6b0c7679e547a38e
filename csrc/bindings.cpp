// Python bindings for the MI355X-native runtime: the C++ block manager and
// the CDNA4 kernel launchers, tensor-checked at this layer.
#include <pybind11/pybind11.h>
#include <torch/extension.h>

#include <c10/hip/HIPStream.h>
#include <hip/hip_runtime.h>

#include <algorithm>
#include <cmath>

#include "attn_inputs.h"
#include "gated_delta.h"
#include "experts.h"
#include "grouped_attn.h"
#include "latent_attn.h"
#include "residual_norm.h"

namespace py = pybind11;

void register_block_manager(py::module_& m);

extern "C" {
void launch_rmsnorm(void*, const void*, const void*, float, int, int, hipStream_t);
void launch_fused_add_rmsnorm(void*, void*, const void*, const void*, float, int, int,
                              hipStream_t);
void launch_swiglu(void*, const void*, int64_t, int, hipStream_t);
void launch_rope_cache(void*, void*, const void*, void*, void*, const int64_t*,
                       const int64_t*, const float*, int, int, int, int, int64_t,
                       int64_t, int64_t, hipStream_t);
void launch_decode_attn(void*, const void*, const void*, const void*, const int*,
                        const int*, float, int, int, int, int, int, int, int64_t,
                        hipStream_t);
void launch_prefill_attn(void*, const void*, const void*, const void*, const int*,
                         const int*, const int*, const int*, const int*, const int*,
                         float, int, int, int, int, int, int, int64_t, hipStream_t);
void launch_sample_fullvocab(int64_t*, const void*, bool, const float*, const int64_t*,
                             const float*, const float*, const uint8_t*, const int32_t*,
                             int, int, hipStream_t);
void launch_sample(int64_t*, const float*, const float*, const int64_t*, const float*,
                   const float*, const uint8_t*, int, int, hipStream_t);
void launch_prefill_attn_mfma(void*, const void*, const void*, const void*, const int*,
                              const int*, const int*, const int*, const int*, const int*,
                              float, int, int, int, int, int, int, int64_t, hipStream_t);
void launch_residual_norm(bool, float*, const void*, const void*, const void*, void*, float,
                          int, int, int64_t, const NormForm*, hipStream_t);
void launch_embed_positions(bool, float*, float*, const int64_t*, const int64_t*, const void*,
                            const float*, float, int, int, int64_t, int64_t, hipStream_t);
void launch_attn_inputs(bool, const AttnInputsArgs*, hipStream_t);
void launch_moe_route(bool, int*, float*, const void*, const void*, const float*, int, int, int,
                      int, int64_t, bool, float, hipStream_t);
void launch_moe_group(int*, int*, int*, int*, const int*, int, int, hipStream_t);
void launch_experts_small(bool, const ExpertsArgs*, int, hipStream_t);
void launch_experts_f32(bool, const ExpertsArgs*, hipStream_t);
void launch_experts_gemm(bool, const ExpertsArgs*, hipStream_t);
void launch_softcap(bool, float*, const void*, float, int64_t, hipStream_t);
bool launch_grouped_decode(const GroupedArgs*, int, int, int, int, hipStream_t);
bool launch_grouped_plain(bool, const GroupedArgs*, int, int, int, hipStream_t);
bool launch_grouped_prefill(const GroupedArgs*, int, int, hipStream_t);
int talk_prefill_tokens(int, int, int, int, int);
bool talk_decode_fits(int, int, int, int);
bool launch_talk_prefill(const GroupedArgs*, int, int, hipStream_t);
bool launch_talk_decode(const GroupedArgs*, int, int, int, hipStream_t);
void launch_cache_keys_values(void*, void*, const void*, const void*, const int64_t*, int, int,
                              int64_t, int, hipStream_t);
void launch_delta_prompts(bool, const DeltaArgs*, int, hipStream_t);
void launch_delta_step(bool, const DeltaArgs*, int, hipStream_t);
void launch_side_gate(bool, float*, const float*, const void*, const void*, const int64_t*, const void*,
                      void*, int, int, int, int64_t, hipStream_t);
void launch_add_to_residual(bool, float*, const void*, void*, int64_t, hipStream_t);
void launch_clamped_glu(bool, void*, const void*, float, float, float, float, int, int, int64_t,
                        int64_t, hipStream_t);
void launch_gelu_gate(bool, void*, const int64_t*, const void*, int, int, int64_t,
                      hipStream_t);
void launch_latent_inputs(bool, void*, const void*, const void*, const int64_t*,
                          const int64_t*, const float*, float, int, int, int, int, int,
                          int64_t, int64_t, void*, const void*, const void*, int, int,
                          int64_t, hipStream_t);
void launch_head_linear(bool, void*, const void*, const void*, const void*, int, int, int,
                        int, int64_t, int, int64_t, int, int64_t, hipStream_t);
bool launch_latent_prefill(const LatentPrefillArgs*, int, int, hipStream_t);
void launch_latent_gather(void*, const void*, const int*, const int*, const int*, const int*,
                          int, int, int, int, int, hipStream_t);
bool launch_latent_attn(bool, bool, const LatentArgs*, int, int, int, int, hipStream_t);
void launch_mfma_probe(float*, const void*, const void*, hipStream_t);
void launch_gemm_bf16(void*, const void*, const void*, int, int, int, hipStream_t);
}

#define CHECK_CUDA(x) TORCH_CHECK(x.is_cuda(), #x " must be a GPU tensor")
#define CHECK_CONT(x) TORCH_CHECK(x.is_contiguous(), #x " must be contiguous")
#define CHECK_BF16(x) TORCH_CHECK(x.scalar_type() == at::kBFloat16, #x " must be bf16")


// q tensors may be strided views into the fused QKV GEMM output: dim-0
// stride is free, heads/dims must be dense
static int64_t q_token_stride(const torch::Tensor& t) {
  TORCH_CHECK(t.stride(2) == 1 && t.stride(1) == t.size(2),
              "head/dim axes must be dense");
  return t.stride(0);
}

static hipStream_t cur_stream() {
  return (hipStream_t)c10::hip::getCurrentHIPStream().stream();
}

static void rmsnorm(torch::Tensor out, torch::Tensor x, torch::Tensor weight,
                    double eps) {
  CHECK_CUDA(x); CHECK_CONT(x); CHECK_BF16(x); CHECK_CONT(out); CHECK_CONT(weight);
  const int h = x.size(-1);
  const int n = x.numel() / h;
  TORCH_CHECK(h % 8 == 0, "hidden size must be a multiple of 8");
  launch_rmsnorm(out.data_ptr(), x.data_ptr(), weight.data_ptr(), (float)eps, n, h,
                 cur_stream());
}

static void fused_add_rmsnorm(torch::Tensor out, torch::Tensor residual,
                              torch::Tensor x, torch::Tensor weight, double eps) {
  CHECK_CUDA(x); CHECK_CONT(x); CHECK_BF16(x); CHECK_CONT(out);
  CHECK_CONT(residual); CHECK_CONT(weight);
  const int h = x.size(-1);
  const int n = x.numel() / h;
  launch_fused_add_rmsnorm(out.data_ptr(), residual.data_ptr(), x.data_ptr(),
                           weight.data_ptr(), (float)eps, n, h, cur_stream());
}

static void swiglu(torch::Tensor out, torch::Tensor gate_up) {
  CHECK_CUDA(gate_up); CHECK_CONT(gate_up); CHECK_BF16(gate_up); CHECK_CONT(out);
  const int inter = gate_up.size(-1) / 2;
  const int64_t n = gate_up.numel() / (2 * inter);
  TORCH_CHECK(inter % 8 == 0, "intermediate size must be a multiple of 8");
  launch_swiglu(out.data_ptr(), gate_up.data_ptr(), n, inter, cur_stream());
}

static void rope_cache(torch::Tensor q, torch::Tensor k, torch::Tensor v,
                       torch::Tensor positions, torch::Tensor slot_mapping,
                       torch::Tensor k_cache, torch::Tensor v_cache,
                       torch::Tensor cos_sin) {
  CHECK_CUDA(q);
  CHECK_CONT(k_cache); CHECK_CONT(v_cache); CHECK_CONT(cos_sin);
  const int64_t q_stride = q_token_stride(q);
  const int64_t kv_stride = q_token_stride(k);
  TORCH_CHECK(v.stride(0) == kv_stride, "k/v must share layout");
  TORCH_CHECK(positions.scalar_type() == at::kLong && slot_mapping.scalar_type() == at::kLong);
  TORCH_CHECK(cos_sin.scalar_type() == at::kFloat);
  const int N = q.size(0);
  const int Hq = q.size(1);
  const int Hkv = k.size(1);
  const int D = q.size(2);
  const int64_t P = cos_sin.size(1);
  TORCH_CHECK(D % 128 == 0 || D <= 512, "head_dim constraint");
  launch_rope_cache(q.data_ptr(), k.data_ptr(), v.data_ptr(), k_cache.data_ptr(),
                    v_cache.data_ptr(), positions.data_ptr<int64_t>(),
                    slot_mapping.data_ptr<int64_t>(), cos_sin.data_ptr<float>(), N,
                    Hq, Hkv, D, P, q_stride, kv_stride, cur_stream());
}

static void decode_attn(torch::Tensor out, torch::Tensor q, torch::Tensor k_cache,
                        torch::Tensor v_cache, torch::Tensor block_tables,
                        torch::Tensor seq_lens, double scale) {
  CHECK_CUDA(q); CHECK_BF16(q); CHECK_CONT(out);
  CHECK_CONT(k_cache); CHECK_CONT(v_cache);
  const int64_t q_stride = q_token_stride(q);
  TORCH_CHECK(block_tables.scalar_type() == at::kInt && seq_lens.scalar_type() == at::kInt);
  CHECK_CONT(block_tables); CHECK_CONT(seq_lens);
  const int B = q.size(0), Hq = q.size(1), D = q.size(2);
  const int Hkv = k_cache.size(2);
  const int kv_block = k_cache.size(1);
  const int max_blocks = block_tables.size(1);
  TORCH_CHECK(D == 128, "decode kernel requires head_dim 128");
  TORCH_CHECK(Hq % Hkv == 0 && Hq / Hkv <= 8, "GQA group must be <= 8");
  launch_decode_attn(out.data_ptr(), q.data_ptr(), k_cache.data_ptr(),
                     v_cache.data_ptr(), block_tables.data_ptr<int>(),
                     seq_lens.data_ptr<int>(), (float)scale, B, Hq, Hkv, D,
                     max_blocks, kv_block, q_stride, cur_stream());
}

static void prefill_attn_impl(torch::Tensor out, torch::Tensor q, torch::Tensor k_cache,
                              torch::Tensor v_cache, torch::Tensor block_tables,
                              torch::Tensor seq_lens, torch::Tensor ctx_lens,
                              torch::Tensor row_starts, torch::Tensor tile_seq,
                              torch::Tensor tile_q0, double scale, bool mfma) {
  CHECK_CUDA(q); CHECK_BF16(q); CHECK_CONT(out);
  const int64_t q_stride = q_token_stride(q);
  TORCH_CHECK(block_tables.scalar_type() == at::kInt);
  const int Hq = q.size(1), D = q.size(2);
  const int Hkv = k_cache.size(2);
  const int kv_block = k_cache.size(1);
  const int max_blocks = block_tables.size(1);
  const int num_tiles = tile_seq.size(0);
  TORCH_CHECK(D == 128, "prefill kernel requires head_dim 128");
  auto fn = mfma ? launch_prefill_attn_mfma : launch_prefill_attn;
  fn(out.data_ptr(), q.data_ptr(), k_cache.data_ptr(),
     v_cache.data_ptr(), block_tables.data_ptr<int>(),
     seq_lens.data_ptr<int>(), ctx_lens.data_ptr<int>(),
     row_starts.data_ptr<int>(), tile_seq.data_ptr<int>(),
     tile_q0.data_ptr<int>(), (float)scale, num_tiles, Hq, Hkv, D,
     max_blocks, kv_block, q_stride, cur_stream());
}

static void prefill_attn(torch::Tensor out, torch::Tensor q, torch::Tensor k_cache,
                         torch::Tensor v_cache, torch::Tensor block_tables,
                         torch::Tensor seq_lens, torch::Tensor ctx_lens,
                         torch::Tensor row_starts, torch::Tensor tile_seq,
                         torch::Tensor tile_q0, double scale) {
  prefill_attn_impl(out, q, k_cache, v_cache, block_tables, seq_lens, ctx_lens,
                    row_starts, tile_seq, tile_q0, scale, /*mfma=*/false);
}

static void prefill_attn_mfma(torch::Tensor out, torch::Tensor q, torch::Tensor k_cache,
                              torch::Tensor v_cache, torch::Tensor block_tables,
                              torch::Tensor seq_lens, torch::Tensor ctx_lens,
                              torch::Tensor row_starts, torch::Tensor tile_seq,
                              torch::Tensor tile_q0, double scale) {
  prefill_attn_impl(out, q, k_cache, v_cache, block_tables, seq_lens, ctx_lens,
                    row_starts, tile_seq, tile_q0, scale, /*mfma=*/true);
}

// C[M,N] = A[M,K] @ B[N,K]^T — the hand-written 256²-tile 8-phase MFMA
// GEMM (csrc/gemm_bf16.hip) for large-M bf16 projections
static void gemm_bf16(torch::Tensor C, torch::Tensor A, torch::Tensor B) {
  CHECK_CUDA(A); CHECK_CONT(A); CHECK_BF16(A);
  CHECK_CONT(B); CHECK_BF16(B); CHECK_CONT(C); CHECK_BF16(C);
  const int M = A.size(0), K = A.size(1), N = B.size(0);
  TORCH_CHECK(B.size(1) == K && C.size(0) == M && C.size(1) == N,
              "gemm_bf16 shape mismatch");
  TORCH_CHECK(K % 128 == 0, "gemm_bf16 requires K % 128 == 0");
  TORCH_CHECK(N % 256 == 0, "gemm_bf16 requires N % 256 == 0");
  launch_gemm_bf16(C.data_ptr(), A.data_ptr(), B.data_ptr(), M, N, K,
                   cur_stream());
}

static torch::Tensor mfma_probe(torch::Tensor a, torch::Tensor b) {
  CHECK_CUDA(a); CHECK_BF16(a); CHECK_CONT(a); CHECK_CONT(b);
  auto d = torch::empty({32, 32}, a.options().dtype(at::kFloat));
  launch_mfma_probe(d.data_ptr<float>(), a.data_ptr(), b.data_ptr(), cur_stream());
  return d;
}

static void sample(torch::Tensor out, torch::Tensor logits, torch::Tensor temps,
                   torch::Tensor top_ks, torch::Tensor top_ps, torch::Tensor uniforms,
                   c10::optional<torch::Tensor> mask) {
  CHECK_CUDA(logits); CHECK_CONT(logits);
  TORCH_CHECK(logits.scalar_type() == at::kFloat);
  const int B = logits.size(0), V = logits.size(1);
  TORCH_CHECK(V <= 512, "sampling kernel supports live vocab <= 512");
  const uint8_t* mptr = nullptr;
  if (mask.has_value()) {
    TORCH_CHECK(mask->scalar_type() == at::kBool && mask->is_contiguous());
    mptr = (const uint8_t*)mask->data_ptr();
  }
  launch_sample(out.data_ptr<int64_t>(), logits.data_ptr<float>(),
                temps.data_ptr<float>(), top_ks.data_ptr<int64_t>(),
                top_ps.data_ptr<float>(), uniforms.data_ptr<float>(), mptr, B, V,
                cur_stream());
}

static void sample_fullvocab(torch::Tensor out, torch::Tensor logits,
                             torch::Tensor temps, torch::Tensor top_ks,
                             torch::Tensor top_ps, torch::Tensor uniforms,
                             c10::optional<torch::Tensor> mask,
                             c10::optional<torch::Tensor> mask_map) {
  CHECK_CUDA(logits); CHECK_CONT(logits);
  const bool bf16 = logits.scalar_type() == at::kBFloat16;
  TORCH_CHECK(bf16 || logits.scalar_type() == at::kFloat,
              "sample_fullvocab wants bf16 or float logits");
  const int B = logits.size(0), V = logits.size(1);
  TORCH_CHECK(V <= (1 << 18), "sample_fullvocab supports vocab <= 256k");
  const uint8_t* mptr = nullptr;
  const int32_t* mapptr = nullptr;
  if (mask.has_value()) {
    TORCH_CHECK(mask->scalar_type() == at::kBool && mask->is_contiguous());
    TORCH_CHECK(mask_map.has_value(), "compact mask needs mask_map");
    TORCH_CHECK(mask_map->scalar_type() == at::kInt && mask_map->is_contiguous());
    TORCH_CHECK(mask_map->numel() == B);
    mptr = (const uint8_t*)mask->data_ptr();
    mapptr = mask_map->data_ptr<int32_t>();
  }
  launch_sample_fullvocab(out.data_ptr<int64_t>(), logits.data_ptr(), bf16,
                          temps.data_ptr<float>(), top_ks.data_ptr<int64_t>(),
                          top_ps.data_ptr<float>(), uniforms.data_ptr<float>(),
                          mptr, mapptr, B, V, cur_stream());
}

// ---- fp32-residual norms, gated activations, latent attention: bf16 or fp32

using OptTensor = c10::optional<torch::Tensor>;

static bool is_bf16(const torch::Tensor& t) {
  TORCH_CHECK(t.scalar_type() == at::kBFloat16 || t.scalar_type() == at::kFloat,
              "want bf16 or fp32");
  return t.scalar_type() == at::kBFloat16;
}

// [rows, k] with dense rows, any row stride
static void check_rows(const torch::Tensor& t, at::ScalarType dtype, int64_t rows,
                       int64_t k) {
  CHECK_CUDA(t);
  TORCH_CHECK(t.dim() == 2 && t.size(0) == rows && t.size(1) == k, "row shape mismatch");
  TORCH_CHECK(t.scalar_type() == dtype, "dtype mismatch");
  TORCH_CHECK(t.size(1) == 1 || t.stride(1) == 1, "rows must be dense");
}

static void check_vec(const torch::Tensor& t, at::ScalarType dtype, int64_t k) {
  CHECK_CUDA(t); CHECK_CONT(t);
  TORCH_CHECK(t.numel() == k && t.scalar_type() == dtype, "vector mismatch");
}

static void check_aligned(const torch::Tensor& t) {
  TORCH_CHECK((uintptr_t)t.data_ptr() % 16 == 0 &&
                  t.stride(0) * t.element_size() % 16 == 0,
              "rows must be 16-byte aligned");
}

static void residual_norm(torch::Tensor x, OptTensor y, OptTensor y_norm, OptTensor x_norm,
                          OptTensor out, double eps, bool center, double offset, double mult,
                          OptTensor states, OptTensor coef, OptTensor partial,
                          int64_t layer, OptTensor x_norm2, OptTensor out2, OptTensor rows,
                          OptTensor weights, OptTensor gate) {
  CHECK_CUDA(x); CHECK_CONT(x);
  TORCH_CHECK(x.scalar_type() == at::kFloat && x.dim() == 2);
  TORCH_CHECK(y || out, "nothing to do");
  const int n = x.size(0), w = x.size(1);
  TORCH_CHECK(w <= 16000, "residual width");  // the row is held in LDS
  const auto dt = y ? y->scalar_type() : out->scalar_type();
  if (y) { check_rows(*y, dt, n, w); CHECK_CONT((*y)); }
  if (y_norm) check_vec(*y_norm, dt, w);
  if (x_norm) check_vec(*x_norm, dt, w);
  if (out) check_rows(*out, dt, n, w);
  NormForm f{};
  f.center = center;
  f.offset = (float)offset;
  f.mult = (float)mult;
  if (rows) {
    TORCH_CHECK(y && weights && rows->dim() == 3, "expert rows");
    f.top = rows->size(1);
    TORCH_CHECK(rows->size(0) == n && rows->size(2) == w && rows->scalar_type() == dt &&
                weights->dim() == 2 && weights->size(0) == n && weights->size(1) == f.top &&
                weights->scalar_type() == at::kFloat, "expert rows");
    CHECK_CUDA((*rows)); CHECK_CONT((*rows)); CHECK_CUDA((*weights)); CHECK_CONT((*weights));
    f.rows = rows->data_ptr();
    f.weights = weights->data_ptr<float>();
  }
  if (gate) {
    TORCH_CHECK(y, "a gate belongs to y");
    check_rows(*gate, dt, n, w);
    f.gate = gate->data_ptr();
    f.gate_stride = gate->stride(0);
  }
  if (out2) {
    TORCH_CHECK(out && x_norm && x_norm2, "second norm");
    check_rows(*out2, dt, n, w); check_vec(*x_norm2, dt, w);
    f.x_norm2 = x_norm2->data_ptr();
    f.out2 = out2->data_ptr();
    f.out2_stride = out2->stride(0);
  }
  if (states) {
    TORCH_CHECK(coef && partial && y, "depth states");
    for (const auto* t : {&*states, &*coef, &*partial}) {
      CHECK_CUDA((*t)); CHECK_CONT((*t));
      TORCH_CHECK(t->scalar_type() == at::kFloat, "depth states are fp32");
    }
    TORCH_CHECK(coef->dim() == 2 && layer >= 0 && layer < coef->size(0) &&
                coef->size(1) >= layer + 2, "depth coefficients");
    TORCH_CHECK(states->dim() == 3 && states->size(0) >= layer + 2 && states->size(1) == n &&
                states->size(2) == w, "depth states");
    TORCH_CHECK(partial->dim() == 3 && partial->size(0) == DEPTH_AHEAD &&
                partial->size(1) == n && partial->size(2) == w, "depth sums");
    const int at = (int)layer % (DEPTH_AHEAD + 1);
    f.n_states = (int)layer + 2;
    f.first = at ? (int)layer - at + 2 : 0;
    f.ready = at - 1;
    f.ahead = std::min(DEPTH_AHEAD, (int)(coef->size(0) - 1 - layer));
    f.states = states->data_ptr<float>();
    f.partial = partial->data_ptr<float>();
    f.coef = coef->data_ptr<float>() + layer * coef->size(1);
    f.coef_stride = coef->size(1);
    f.plane = (int64_t)n * w;
  }
  if (n == 0) return;
  launch_residual_norm(is_bf16(y ? *y : *out), x.data_ptr<float>(),
                       y ? y->data_ptr() : nullptr, y_norm ? y_norm->data_ptr() : nullptr,
                       x_norm ? x_norm->data_ptr() : nullptr,
                       out ? out->data_ptr() : nullptr, (float)eps, n, w,
                       out ? out->stride(0) : w, &f, cur_stream());
}

static void check_ids(const torch::Tensor& t, int64_t n) {
  CHECK_CUDA(t); CHECK_CONT(t);
  TORCH_CHECK(t.scalar_type() == at::kLong && t.numel() == n, "want int64 per row");
}

static void embed_positions(torch::Tensor x, OptTensor copy, torch::Tensor token_ids,
                            torch::Tensor positions, torch::Tensor table, OptTensor cos_sin,
                            double scale) {
  const int n = x.size(0), w = x.size(1);
  check_rows(x, at::kFloat, n, w); CHECK_CONT(x);
  if (copy) { check_rows(*copy, at::kFloat, n, w); CHECK_CONT((*copy)); }
  check_ids(token_ids, n); check_ids(positions, n);
  check_rows(table, table.scalar_type(), table.size(0), w); CHECK_CONT(table);
  if (cos_sin) {
    CHECK_CUDA((*cos_sin)); CHECK_CONT((*cos_sin));
    TORCH_CHECK(cos_sin->scalar_type() == at::kFloat && cos_sin->dim() == 3 &&
                cos_sin->size(0) == 2 && cos_sin->size(2) == (w + 1) / 2, "position table");
  }
  if (n == 0) return;
  launch_embed_positions(is_bf16(table), x.data_ptr<float>(),
                         copy ? copy->data_ptr<float>() : nullptr,
                         token_ids.data_ptr<int64_t>(), positions.data_ptr<int64_t>(),
                         table.data_ptr(), cos_sin ? cos_sin->data_ptr<float>() : nullptr,
                         (float)scale, n, w, table.size(0), cos_sin ? cos_sin->size(1) : 1, cur_stream());
}

static void softcap(torch::Tensor out, torch::Tensor x, double cap) {
  CHECK_CUDA(x); CHECK_CONT(x); CHECK_CUDA(out); CHECK_CONT(out);
  TORCH_CHECK(out.scalar_type() == at::kFloat && out.numel() == x.numel() && cap > 0);
  if (x.numel() == 0) return;
  launch_softcap(is_bf16(x), out.data_ptr<float>(), x.data_ptr(), (float)cap, x.numel(),
                 cur_stream());
}

// x_out = x + y; s = gelu_tanh(gate x_out) * table[token, offset:]
static void side_gate(torch::Tensor s, torch::Tensor x_out, torch::Tensor x, torch::Tensor y, torch::Tensor gate,
                      torch::Tensor token_ids, torch::Tensor table, int64_t offset) {
  const int n = x.size(0), w = x.size(1), dim = s.size(1);
  CHECK_CUDA(x); CHECK_CONT(x); CHECK_CUDA(x_out); CHECK_CONT(x_out);
  TORCH_CHECK(x.scalar_type() == at::kFloat && x_out.scalar_type() == at::kFloat &&
              x_out.sizes() == x.sizes() && x_out.data_ptr() != x.data_ptr());
  const auto dt = y.scalar_type();
  check_rows(y, dt, n, w); CHECK_CONT(y);
  check_rows(s, dt, n, dim); CHECK_CONT(s);
  check_rows(gate, dt, dim, w); CHECK_CONT(gate);
  check_rows(table, dt, table.size(0), table.size(1));
  CHECK_CUDA(token_ids); CHECK_CONT(token_ids);
  TORCH_CHECK(token_ids.scalar_type() == at::kLong && token_ids.numel() == n);
  TORCH_CHECK(offset >= 0 && offset + dim <= table.size(1), "table columns");
  TORCH_CHECK(w % 8 == 0 && w <= 16000, "residual width");
  if (n == 0) return;
  launch_side_gate(is_bf16(y), x_out.data_ptr<float>(), x.data_ptr<float>(), y.data_ptr(), gate.data_ptr(),
                   token_ids.data_ptr<int64_t>(),
                   (const char*)table.data_ptr() + offset * table.element_size(),
                   s.data_ptr(), n, w, dim, table.stride(0), cur_stream());
}

static void add_to_residual(torch::Tensor x, torch::Tensor y, OptTensor out) {
  CHECK_CUDA(x); CHECK_CONT(x); CHECK_CUDA(y); CHECK_CONT(y);
  TORCH_CHECK(x.scalar_type() == at::kFloat && x.numel() == y.numel());
  if (out) {
    CHECK_CUDA((*out)); CHECK_CONT((*out));
    TORCH_CHECK(out->scalar_type() == y.scalar_type() && out->numel() == x.numel());
  }
  if (x.numel() == 0) return;
  launch_add_to_residual(is_bf16(y), x.data_ptr<float>(), y.data_ptr(),
                         out ? out->data_ptr() : nullptr, x.numel(), cur_stream());
}

static void clamped_glu(torch::Tensor out, torch::Tensor gate_up, double limit,
                        double alpha, double offset, double cubic) {
  const int rows = out.size(0), inter = out.size(1);
  check_rows(out, gate_up.scalar_type(), rows, inter);
  check_rows(gate_up, gate_up.scalar_type(), rows, 2 * (int64_t)inter);
  check_aligned(out); check_aligned(gate_up);
  TORCH_CHECK(inter % 8 == 0, "padded width must be a multiple of 8");
  if (rows == 0) return;
  launch_clamped_glu(is_bf16(out), out.data_ptr(), gate_up.data_ptr(), (float)limit,
                     (float)alpha, (float)offset, (float)cubic, rows, inter, gate_up.stride(0),
                     out.stride(0), cur_stream());
}

static void gelu_gate(torch::Tensor s, torch::Tensor token_ids, torch::Tensor table,
                      int64_t offset) {
  const int rows = s.size(0), dim = s.size(1);
  check_rows(s, s.scalar_type(), rows, dim); CHECK_CONT(s);
  check_rows(table, s.scalar_type(), table.size(0), table.size(1));
  CHECK_CUDA(token_ids); CHECK_CONT(token_ids);
  TORCH_CHECK(token_ids.scalar_type() == at::kLong && token_ids.numel() == rows);
  TORCH_CHECK(offset >= 0 && offset + dim <= table.size(1), "table columns");
  if (rows == 0) return;
  launch_gelu_gate(is_bf16(s), s.data_ptr(), token_ids.data_ptr<int64_t>(),
                   (const char*)table.data_ptr() + offset * table.element_size(), rows, dim,
                   table.stride(0), cur_stream());
}

static void check_rotation(const torch::Tensor& cos_sin, const torch::Tensor& positions,
                           int64_t n, int64_t rot_dim) {
  CHECK_CUDA(cos_sin); CHECK_CONT(cos_sin); CHECK_CUDA(positions); CHECK_CONT(positions);
  TORCH_CHECK(cos_sin.scalar_type() == at::kFloat && cos_sin.dim() == 3 &&
              cos_sin.size(0) == 2 && cos_sin.size(2) * 2 == rot_dim, "rotation table");
  TORCH_CHECK(positions.scalar_type() == at::kLong && positions.numel() == n);
}

// Cache rows of kv, and cq = rmsnorm(q) over q's first q_rank columns (low-rank
// queries; q, q_norm and cq come together).
static void latent_inputs(torch::Tensor cache, torch::Tensor kv, torch::Tensor norm_w,
                          torch::Tensor positions, torch::Tensor slots,
                          torch::Tensor cos_sin, double eps, int64_t kv_rank,
                          int64_t rot_dim, int64_t rank, OptTensor cq, OptTensor q,
                          OptTensor q_norm, int64_t q_rank) {
  const int n = kv.size(0);
  check_rows(kv, kv.scalar_type(), n, kv_rank + rot_dim);
  check_vec(norm_w, kv.scalar_type(), kv_rank);
  check_rotation(cos_sin, positions, n, rot_dim);
  CHECK_CUDA(slots); CHECK_CONT(slots); CHECK_CUDA(cache); CHECK_CONT(cache);
  TORCH_CHECK(slots.scalar_type() == at::kLong && slots.numel() == n);
  TORCH_CHECK(cache.scalar_type() == kv.scalar_type());
  const int row = cache.size(-1);
  TORCH_CHECK(kv_rank <= rank && rank + rot_dim <= row && (row - rank) % 2 == 0);
  int k = 0;
  if (q) {
    TORCH_CHECK(cq && q_norm, "low-rank query");
    k = q->size(1);
    check_rows(*q, kv.scalar_type(), n, k); check_aligned(*q);
    check_rows(*cq, kv.scalar_type(), n, k); CHECK_CONT((*cq));
    check_vec(*q_norm, kv.scalar_type(), k);
    TORCH_CHECK(k % 8 == 0 && q_rank > 0 && q_rank <= k);
  }
  if (n == 0) return;
  launch_latent_inputs(is_bf16(kv), cache.data_ptr(), kv.data_ptr(), norm_w.data_ptr(),
                       positions.data_ptr<int64_t>(), slots.data_ptr<int64_t>(),
                       cos_sin.data_ptr<float>(), (float)eps, n, kv_rank, rot_dim, rank, row,
                       kv.stride(0), cos_sin.size(1), q ? cq->data_ptr() : nullptr,
                       q ? q->data_ptr() : nullptr, q ? q_norm->data_ptr() : nullptr, k,
                       (int)q_rank, q ? q->stride(0) : 0, cur_stream());
}

// [N, H, K] with dense vectors, any token and head stride
static void check_heads(const torch::Tensor& t, at::ScalarType dtype, int64_t n, int64_t h) {
  CHECK_CUDA(t);
  TORCH_CHECK(t.dim() == 3 && t.size(0) == n && t.size(1) == h && t.stride(2) == 1,
              "head shape mismatch");
  TORCH_CHECK(t.scalar_type() == dtype, "dtype mismatch");
  check_aligned(t);
  TORCH_CHECK(t.stride(1) * t.element_size() % 16 == 0, "heads must be 16-byte aligned");
}

static void head_linear(torch::Tensor out, torch::Tensor x, torch::Tensor w,
                        OptTensor gate) {
  const int n = x.size(0), h = x.size(1), k = x.size(2), o = out.size(2);
  check_heads(x, w.scalar_type(), n, h);
  check_heads(out, w.scalar_type(), n, h);
  CHECK_CUDA(w); CHECK_CONT(w);
  TORCH_CHECK(w.dim() == 3 && w.size(0) == h && w.size(1) == o && w.size(2) == k);
  TORCH_CHECK(k % 32 == 0 && o % 32 == 0, "head_linear wants multiples of 32");
  if (gate) check_rows(*gate, w.scalar_type(), n, h);
  if (n == 0) return;
  launch_head_linear(is_bf16(w), out.data_ptr(), x.data_ptr(), w.data_ptr(),
                     gate ? gate->data_ptr() : nullptr, n, h, o, k, x.stride(0), x.stride(1),
                     out.stride(0), out.stride(1), gate ? gate->stride(0) : 0, cur_stream());
}

static const int* opt_int(const OptTensor& t, int64_t n) {
  if (!t) return nullptr;
  CHECK_CUDA((*t)); CHECK_CONT((*t));
  TORCH_CHECK(t->scalar_type() == at::kInt && t->numel() == n);
  return t->data_ptr<int>();
}

// q [tokens, H, rank] absorbed, q_rot [tokens, H, rot] -> out [tokens, H, rank].  Prefill chunks bring ctx_lens,
// row_starts and tiles; decode (one token per table row) brings none of them.
static void latent_attn(torch::Tensor out, torch::Tensor q, torch::Tensor q_rot,
                        torch::Tensor cos_sin, int64_t rot_dim, torch::Tensor cache,
                        torch::Tensor tables, torch::Tensor seq_lens, OptTensor ctx_lens,
                        OptTensor row_starts, OptTensor tile_seq, OptTensor tile_r0,
                        OptTensor part, OptTensor part_ml, OptTensor sink, double scale,
                        int64_t window, int64_t mg, int64_t n_split, bool mfma) {
  CHECK_CUDA(q); CHECK_CONT(q); CHECK_CONT(out); CHECK_CUDA(cache); CHECK_CONT(cache);
  CHECK_CUDA(tables); CHECK_CONT(tables); CHECK_CUDA(seq_lens); CHECK_CONT(seq_lens);
  const bool bf16 = is_bf16(q);
  const int tokens = q.size(0), H = q.size(1), rank = q.size(2);
  const int row = rank + q_rot.size(2);
  TORCH_CHECK(out.sizes() == q.sizes());
  check_heads(q_rot, q.scalar_type(), tokens, H);
  CHECK_CUDA(cos_sin); CHECK_CONT(cos_sin);
  TORCH_CHECK(cos_sin.scalar_type() == at::kFloat && cos_sin.dim() == 3 &&
              cos_sin.size(0) == 2 && cos_sin.size(2) * 2 == rot_dim &&
              rot_dim <= q_rot.size(2), "rotation table");
  TORCH_CHECK(cache.dim() == 3 && cache.size(2) == row);
  TORCH_CHECK(cache.scalar_type() == q.scalar_type() && out.scalar_type() == q.scalar_type());
  TORCH_CHECK(tables.scalar_type() == at::kInt && seq_lens.scalar_type() == at::kInt);
  const int seqs = tables.size(0);
  TORCH_CHECK(seq_lens.numel() == seqs);
  TORCH_CHECK(!mfma || (bf16 && row - rank == 64), "no MFMA kernel for this row");
  TORCH_CHECK(window > 0 && n_split >= 1 && n_split <= 64 && (mfma || n_split == 1));
  TORCH_CHECK(mg == 1 || mg == 2 || (mg == 4 && rank <= 256) || !mfma, "row tile");
  const int per_tile = mfma ? 16 * (int)mg : 1;
  int tiles;
  if (tile_seq) {
    TORCH_CHECK(tile_r0 && ctx_lens && row_starts, "prefill metadata");
    tiles = tile_seq->numel();
  } else {
    TORCH_CHECK(tokens == seqs, "decode has one token per sequence");
    tiles = seqs * ((H + per_tile - 1) / per_tile);
  }
  if (tiles == 0) return;
  LatentArgs a{};
  a.out = out.data_ptr();
  if (n_split > 1) {
    TORCH_CHECK(part && part_ml && part->is_contiguous() && part_ml->is_contiguous());
    TORCH_CHECK(part->scalar_type() == at::kFloat && part_ml->scalar_type() == at::kFloat);
    TORCH_CHECK(part->numel() >= n_split * tokens * H * rank &&
                part_ml->numel() >= 2 * n_split * tokens * H, "split workspace");
    a.part = part->data_ptr<float>();
    a.part_ml = (float2*)part_ml->data_ptr<float>();
  }
  a.q = q.data_ptr();
  a.q_rot = q_rot.data_ptr();
  a.rot_token = q_rot.stride(0);
  a.rot_head = q_rot.stride(1);
  a.rot_dim = (int)rot_dim;
  a.cos_sin = cos_sin.data_ptr<float>();
  a.positions = cos_sin.size(1);
  a.cache = cache.data_ptr();
  if (sink) { check_vec(*sink, at::kFloat, H); a.sink = sink->data_ptr<float>(); }
  a.tables = tables.data_ptr<int>();
  a.seq_lens = seq_lens.data_ptr<int>();
  a.ctx_lens = opt_int(ctx_lens, seqs);
  a.row_starts = opt_int(row_starts, seqs);
  a.tile_seq = opt_int(tile_seq, tiles);
  a.tile_r0 = opt_int(tile_r0, tiles);
  a.H = H;
  a.max_blocks = tables.size(1);
  a.kv_block = cache.size(1);
  a.window = (int)window;
  a.n_split = (int)n_split;
  a.rows = tokens * H;
  a.scale = (float)scale;
  TORCH_CHECK(launch_latent_attn(bf16, mfma, &a, rank, row, (int)mg, tiles, cur_stream()),
              "latent attention: unsupported sizes rank ", rank, " row ", row);
}

// rows of out: sequence s's cached rows from position first[s] on, at starts[s]
static void latent_gather(torch::Tensor out, torch::Tensor cache, torch::Tensor tables,
                          torch::Tensor seq_lens, torch::Tensor first, torch::Tensor starts,
                          int64_t max_keys) {
  CHECK_CUDA(out); CHECK_CONT(out); CHECK_BF16(out);
  CHECK_CUDA(cache); CHECK_CONT(cache); CHECK_BF16(cache);
  CHECK_CUDA(tables); CHECK_CONT(tables);
  TORCH_CHECK(tables.scalar_type() == at::kInt);
  const int seqs = tables.size(0), row = cache.size(2);
  TORCH_CHECK(out.size(1) == row && row % 8 == 0);
  if (seqs == 0 || max_keys == 0) return;
  launch_latent_gather(out.data_ptr(), cache.data_ptr(), tables.data_ptr<int>(),
                       opt_int(seq_lens, seqs), opt_int(first, seqs), opt_int(starts, seqs),
                       seqs, max_keys, row, tables.size(1), cache.size(1), cur_stream());
}

// q [tokens, H, d + 64], kv [keys, H * (d + v)], k_rot [keys, 64], gate [tokens, H]
// -> out [tokens, H, v]; rows of sequences without tiles are left alone.
static void latent_prefill(torch::Tensor out, torch::Tensor q, torch::Tensor kv,
                           torch::Tensor k_rot, OptTensor gate, torch::Tensor cos_sin,
                           int64_t rot_dim, torch::Tensor seq_lens, torch::Tensor ctx_lens,
                           torch::Tensor row_starts, torch::Tensor tile_seq,
                           torch::Tensor tile_q0, torch::Tensor key_first,
                           torch::Tensor key_starts, OptTensor sink, double scale,
                           int64_t window) {
  const int tokens = q.size(0), H = q.size(1), d = q.size(2) - 64, v = out.size(2);
  check_heads(q, at::kBFloat16, tokens, H);
  check_heads(out, at::kBFloat16, tokens, H);
  TORCH_CHECK(q.stride(1) == d + 64 && out.stride(1) == v, "heads must be dense");
  const int64_t keys = kv.size(0);
  check_rows(kv, at::kBFloat16, keys, (int64_t)H * (d + v)); check_aligned(kv);
  check_rows(k_rot, at::kBFloat16, keys, 64); check_aligned(k_rot);
  if (gate) check_rows(*gate, at::kBFloat16, tokens, H);
  CHECK_CUDA(cos_sin); CHECK_CONT(cos_sin);
  TORCH_CHECK(cos_sin.scalar_type() == at::kFloat && cos_sin.dim() == 3 &&
              cos_sin.size(0) == 2 && cos_sin.size(2) * 2 == rot_dim && rot_dim <= 64,
              "rotation table");
  TORCH_CHECK(window > 0);
  const int seqs = seq_lens.numel();
  LatentPrefillArgs a{};
  a.out = out.data_ptr();
  a.q = q.data_ptr();
  a.kv = kv.data_ptr();
  a.k_rot = k_rot.data_ptr();
  a.gate = gate ? gate->data_ptr() : nullptr;
  if (sink) { check_vec(*sink, at::kFloat, H); a.sink = sink->data_ptr<float>(); }
  a.cos_sin = cos_sin.data_ptr<float>();
  a.n_tiles = tile_seq.numel();
  a.seq_lens = opt_int(seq_lens, seqs);
  a.ctx_lens = opt_int(ctx_lens, seqs);
  a.row_starts = opt_int(row_starts, seqs);
  a.tile_seq = opt_int(tile_seq, a.n_tiles);
  a.tile_q0 = opt_int(tile_q0, a.n_tiles);
  a.key_first = opt_int(key_first, seqs);
  a.key_starts = opt_int(key_starts, seqs);
  a.out_stride = out.stride(0);
  a.q_stride = q.stride(0);
  a.kv_stride = kv.stride(0);
  a.rot_stride = k_rot.stride(0);
  a.gate_stride = gate ? gate->stride(0) : 0;
  a.positions = cos_sin.size(1);
  a.H = H;
  a.rot_dim = (int)rot_dim;
  a.window = (int)window;
  a.scale = (float)scale;
  if (a.n_tiles == 0) return;
  TORCH_CHECK(launch_latent_prefill(&a, d, v, cur_stream()),
              "latent prefill: unsupported sizes d ", d, " v ", v);
}

// ---- grouped attention, delta rule

// [N, heads, size] with dense heads and vectors, any token stride, 16-byte aligned
static void check_token_heads(const torch::Tensor& t, at::ScalarType dtype, int64_t n,
                              int64_t heads, int64_t size) {
  CHECK_CUDA(t);
  TORCH_CHECK(t.dim() == 3 && t.size(0) == n && t.size(1) == heads && t.size(2) == size,
              "head shape mismatch");
  TORCH_CHECK(t.stride(2) == 1 && (heads == 1 || t.stride(1) == size), "heads must be dense");
  TORCH_CHECK(t.scalar_type() == dtype, "dtype mismatch");
  check_aligned(t);
}

static void check_cache(const torch::Tensor& t, at::ScalarType dtype) {
  CHECK_CUDA(t); CHECK_CONT(t);
  TORCH_CHECK(t.dim() == 4 && t.scalar_type() == dtype, "cache layout");
  TORCH_CHECK(t.size(3) * t.element_size() % 16 == 0, "cache rows must be 16-byte multiples");
}

static void cache_keys_values(torch::Tensor k_cache, torch::Tensor v_cache, torch::Tensor k,
                              torch::Tensor v, torch::Tensor slots) {
  const auto dt = k.scalar_type();
  const int n = k.size(0), G = k.size(1);
  check_cache(k_cache, dt); check_cache(v_cache, dt);
  check_token_heads(k, dt, n, G, k_cache.size(3));
  check_token_heads(v, dt, n, G, v_cache.size(3));
  TORCH_CHECK(k_cache.size(2) == G && v_cache.size(2) == G && k_cache.size(0) == v_cache.size(0) &&
              k_cache.size(1) == v_cache.size(1), "cache shapes");
  TORCH_CHECK(k.stride(0) == v.stride(0), "k and v must share a row stride");
  check_ids(slots, n);
  if (n == 0) return;
  const int unit = 16 / (int)k.element_size();
  launch_cache_keys_values(k_cache.data_ptr(), v_cache.data_ptr(), k.data_ptr(), v.data_ptr(),
                           slots.data_ptr<int64_t>(), G * k.size(2) / unit, G * v.size(2) / unit,
                           k.stride(0) / unit, n, cur_stream());
}

// q [tokens, H, d] -> out [tokens, H, v].  Prefill chunks bring ctx_lens, row_starts and
// tiles; decode (one token per table row) brings none of them.
// kind: 0 plain, 1 decode, 2 prefill on the matrix cores, with mixed scores 3 decode, 4 prefill
static void grouped_attn(torch::Tensor out, torch::Tensor q, torch::Tensor k_cache,
                         torch::Tensor v_cache, torch::Tensor tables, torch::Tensor seq_lens,
                         OptTensor ctx_lens, OptTensor row_starts, OptTensor tile_seq,
                         OptTensor tile_q0, OptTensor sink, OptTensor bias, OptTensor gate,
                         OptTensor talk, OptTensor part, OptTensor part_ml, double scale,
                         double cap, int64_t window, int64_t chunk, int64_t keep, bool sigmoid,
                         int64_t kind, int64_t gm, int64_t n_split) {
  const auto dt = q.scalar_type();
  const bool bf16 = is_bf16(q);
  const int tokens = q.size(0), H = q.size(1), d = q.size(2), v = out.size(2);
  check_token_heads(q, dt, tokens, H, d);
  check_token_heads(out, dt, tokens, H, v);
  check_cache(k_cache, dt); check_cache(v_cache, dt);
  const int G = k_cache.size(2);
  TORCH_CHECK(k_cache.size(3) == d && v_cache.size(3) == v && v_cache.size(2) == G &&
              k_cache.size(0) == v_cache.size(0) && k_cache.size(1) == v_cache.size(1) &&
              H % G == 0, "cache shapes");
  CHECK_CUDA(tables); CHECK_CONT(tables);
  TORCH_CHECK(tables.scalar_type() == at::kInt && tables.dim() == 2);
  const int seqs = tables.size(0);
  TORCH_CHECK(window > 0 && keep >= 0 && cap >= 0 && n_split >= 1 && n_split <= 64);
  TORCH_CHECK(chunk > 0 && chunk <= (1 << 30) && (keep == 0 || chunk == (1 << 30)),
              "chunks keep no first tokens");
  TORCH_CHECK(kind == 0 || bf16, "the matrix-core kernels take bf16");
  const bool decode = kind == 1 || kind == 3, prefill = kind == 2 || kind == 4;
  TORCH_CHECK(decode || n_split == 1, "only decode splits keys");
  TORCH_CHECK(prefill <= (bool)tile_seq && !(decode && tile_seq), "tiles");
  if (tokens == 0 || seqs == 0) return;
  GroupedArgs a{};
  a.out = out.data_ptr();
  if (n_split > 1) {
    TORCH_CHECK(part && part_ml && part->is_contiguous() && part_ml->is_contiguous());
    TORCH_CHECK(part->scalar_type() == at::kFloat && part_ml->scalar_type() == at::kFloat);
    TORCH_CHECK(part->numel() >= n_split * tokens * H * v &&
                part_ml->numel() >= 2 * n_split * tokens * H, "split workspace");
    a.part = part->data_ptr<float>();
    a.part_ml = (float2*)part_ml->data_ptr<float>();
  }
  a.q = q.data_ptr();
  a.k_cache = k_cache.data_ptr();
  a.v_cache = v_cache.data_ptr();
  if (sink) { check_vec(*sink, at::kFloat, H); a.sink = sink->data_ptr<float>(); }
  TORCH_CHECK(!(sink && sigmoid), "a sink belongs to the softmax");
  if (bias) {
    TORCH_CHECK(bias->dim() == 2 && bias->size(0) == H && bias->size(1) > 0 &&
                bias->scalar_type() == at::kFloat, "bias by head and distance");
    CHECK_CUDA((*bias)); CHECK_CONT((*bias));
    a.bias = bias->data_ptr<float>();
    a.n_bias = bias->size(1);
  }
  if (gate) {
    check_rows(*gate, dt, tokens, H);
    a.gate = gate->data_ptr();
    a.gate_stride = gate->stride(0);
  }
  if (talk) {
    check_rows(*talk, at::kFloat, H, H); CHECK_CONT((*talk));
    a.talk = talk->data_ptr<float>();
  }
  a.chunk = (int)chunk;
  a.sigmoid = sigmoid;
  a.out_stride = out.stride(0);
  a.tables = tables.data_ptr<int>();
  a.seq_lens = opt_int(seq_lens, seqs);
  a.ctx_lens = opt_int(ctx_lens, seqs);
  a.row_starts = opt_int(row_starts, seqs);
  if (tile_seq) {
    TORCH_CHECK(ctx_lens && row_starts && tile_q0, "prefill metadata");
    a.n_tiles = tile_seq->numel();
    TORCH_CHECK(prefill || a.n_tiles == tokens, "the plain kernel takes a token per tile");
  } else {
    TORCH_CHECK(tokens == seqs, "decode has one token per sequence");
  }
  a.tile_seq = opt_int(tile_seq, a.n_tiles);
  a.tile_q0 = opt_int(tile_q0, a.n_tiles);
  a.q_stride = q.stride(0);
  a.H = H;
  a.G = G;
  a.max_blocks = tables.size(1);
  a.kv_block = k_cache.size(1);
  a.window = (int)window;
  a.keep = (int)keep;
  a.n_split = (int)n_split;
  a.rows = tokens * H;
  a.scale = (float)scale;
  a.cap = (float)cap;
  TORCH_CHECK((bool)talk ? kind != 1 && kind != 2 : kind < 3, "mixed scores");
  const bool ok = kind == 4   ? launch_talk_prefill(&a, d, v, cur_stream())
                  : kind == 3 ? launch_talk_decode(&a, d, v, seqs, cur_stream())
                  : kind == 2   ? launch_grouped_prefill(&a, d, v, cur_stream())
                  : kind == 1 ? launch_grouped_decode(&a, d, v, seqs, (int)gm, cur_stream())
                              : launch_grouped_plain(bf16, &a, d, v, tokens, cur_stream());
  TORCH_CHECK(ok, "grouped attention: unsupported sizes d ", d, " v ", v);
}

// proj [N, (H + G) d + G v] -> q [N, H, d] and the rows' cache slots.  back, states: per row;
// ring_rows: rows that join the ring after all others have read it.
static void attention_inputs(torch::Tensor q, torch::Tensor k_cache, torch::Tensor v_cache,
                             torch::Tensor proj, torch::Tensor positions, torch::Tensor slots,
                             int64_t dim, int64_t vdim, double eps, OptTensor conv,
                             OptTensor ring, OptTensor back, OptTensor states,
                             OptTensor ring_rows, bool write_ring, OptTensor q_norm,
                             OptTensor k_norm, bool v_norm, OptTensor cos_sin,
                             OptTensor head_mult, double q_coef, double q_every) {
  const auto dt = proj.scalar_type();
  const bool bf16 = is_bf16(proj);
  AttnInputsArgs a{};
  a.N = q.size(0);
  a.H = q.size(1);
  a.d = q.size(2);
  check_token_heads(q, dt, a.N, a.H, a.d); CHECK_CONT(q);
  check_cache(k_cache, dt); check_cache(v_cache, dt);
  a.G = k_cache.size(2);
  a.v = v_cache.size(3);
  TORCH_CHECK(k_cache.size(3) == a.d && v_cache.size(2) == a.G &&
              k_cache.size(0) == v_cache.size(0) && k_cache.size(1) == v_cache.size(1),
              "cache shapes");
  a.C = (a.H + a.G) * a.d + a.G * a.v;
  check_rows(proj, dt, a.N, a.C); check_aligned(proj);
  check_ids(positions, a.N); check_ids(slots, a.N);
  TORCH_CHECK(dim > 0 && dim <= a.d && vdim > 0 && vdim <= a.v && a.d % 8 == 0 && a.v % 8 == 0,
              "head sizes");
  if (conv) {
    a.taps = conv->size(0);
    TORCH_CHECK(a.taps > 0 && ring && states, "convolution state");
    check_rows(*conv, dt, a.taps, a.C); CHECK_CONT((*conv));
    CHECK_CUDA((*ring)); CHECK_CONT((*ring));
    TORCH_CHECK(ring->dim() == 3 && ring->size(1) == a.taps && ring->size(2) == a.C &&
                ring->scalar_type() == dt, "convolution state");
    a.conv = conv->data_ptr();
    a.ring = ring->data_ptr();
    a.back = opt_int(back, a.N);
    a.states = opt_int(states, a.N);
    a.write_ring = write_ring;
    if (ring_rows) {
      a.n_ring_rows = ring_rows->numel();
      a.ring_rows = opt_int(ring_rows, a.n_ring_rows);
      TORCH_CHECK(a.n_ring_rows <= 65535, "grid");
    }
  }
  if (q_norm) {
    TORCH_CHECK(k_norm, "q and k are normed alike");
    // weights of all heads: a norm over all heads
    a.row_norm = q_norm->numel() != a.d;
    check_vec(*q_norm, dt, (a.row_norm ? a.H : 1) * a.d);
    check_vec(*k_norm, dt, (a.row_norm ? a.G : 1) * a.d);
    TORCH_CHECK(!a.row_norm || (!conv && !v_norm && a.C <= 16 * 1024 * (bf16 ? 8 : 4)),
                "norms over all heads");
    a.q_norm = q_norm->data_ptr();
    a.k_norm = k_norm->data_ptr();
  }
  a.v_norm = v_norm;
  if (cos_sin) {
    check_rotation(*cos_sin, positions, a.N, 2 * cos_sin->size(2));
    a.pairs = cos_sin->size(2);
    TORCH_CHECK(2 * a.pairs <= a.d, "rotated dimensions");
    a.cos_sin = cos_sin->data_ptr<float>();
    a.P = cos_sin->size(1);
  }
  if (head_mult) {
    check_vec(*head_mult, at::kFloat, a.H);
    a.head_mult = head_mult->data_ptr<float>();
  }
  TORCH_CHECK(q_every >= 0);
  a.q_coef = (float)q_coef;
  a.q_every = (float)q_every;
  a.q = q.data_ptr();
  a.k_cache = k_cache.data_ptr();
  a.v_cache = v_cache.data_ptr();
  a.proj = proj.data_ptr();
  a.positions = positions.data_ptr<int64_t>();
  a.slots = slots.data_ptr<int64_t>();
  a.stride = proj.stride(0);
  a.dim = (int)dim;
  a.vdim = (int)vdim;
  a.eps = (float)eps;
  TORCH_CHECK(a.N <= 65535, "grid");
  if (a.N == 0) return;
  launch_attn_inputs(bf16, &a, cur_stream());
}

// ---- mixture of experts

static void moe_route(torch::Tensor ids, torch::Tensor weights, torch::Tensor h, torch::Tensor w,
                      OptTensor bias, bool sigmoid, double scale) {
  const int N = h.size(0), K = h.size(1), E = w.size(0), top = ids.size(1);
  check_rows(h, h.scalar_type(), N, K); check_aligned(h);
  check_rows(w, h.scalar_type(), E, K); CHECK_CONT(w);
  check_rows(ids, at::kInt, N, top); CHECK_CONT(ids);
  check_rows(weights, at::kFloat, N, top); CHECK_CONT(weights);
  if (bias) check_vec(*bias, at::kFloat, E);
  TORCH_CHECK(K % 64 == 0 && E <= 512 && top > 0 && top <= E && top <= 64, "router sizes");
  if (N == 0) return;
  launch_moe_route(is_bf16(h), ids.data_ptr<int>(), weights.data_ptr<float>(), h.data_ptr(),
                   w.data_ptr(), bias ? bias->data_ptr<float>() : nullptr, N, E, K, top,
                   h.stride(0), sigmoid, (float)scale, cur_stream());
}

// perm [n], offsets [E + 2]; tiles of EXPERT_TILE rows: at most ceil(n / tile) + E
static void moe_group(torch::Tensor perm, torch::Tensor offsets, OptTensor tile_expert,
                      OptTensor tile_row, torch::Tensor ids, int64_t E) {
  const int64_t n = ids.numel();
  CHECK_CUDA(ids); CHECK_CONT(ids);
  TORCH_CHECK(ids.scalar_type() == at::kInt && E > 0 && E <= 512 && n < (1 << 30));
  const int64_t tiles = tile_expert ? n / EXPERT_TILE + E : 0;
  int* te = (int*)opt_int(tile_expert, tiles);
  int* tr = (int*)opt_int(tile_row, tiles);
  TORCH_CHECK(!te == !tr, "tiles");
  launch_moe_group((int*)opt_int(perm, n), (int*)opt_int(offsets, E + 2), te, tr,
                   ids.data_ptr<int>(), (int)n, (int)E, cur_stream());
}

// One product of the routed experts (experts.h).  kind: 0 fp32, 1 few rows, 2 tiles
static void experts_linear(torch::Tensor out, torch::Tensor x, torch::Tensor w, torch::Tensor ids,
                           OptTensor perm, OptTensor offsets, OptTensor tile_expert,
                           OptTensor tile_row, bool glu, double limit, double alpha,
                           double offset, double cubic, int64_t kind, int64_t tt) {
  const auto dt = x.scalar_type();
  ExpertsArgs a{};
  CHECK_CUDA(w); CHECK_CONT(w); CHECK_CUDA(ids); CHECK_CONT(ids);
  TORCH_CHECK(w.dim() == 3 && w.scalar_type() == dt && ids.dim() == 2 &&
              ids.scalar_type() == at::kInt, "experts");
  a.entries = ids.numel();
  a.top = ids.size(1);
  a.E = w.size(0);
  a.O = (int)(glu ? w.size(1) / 2 : w.size(1));
  a.K = w.size(2);
  check_rows(x, dt, glu ? ids.size(0) : a.entries, a.K); check_aligned(x);
  check_rows(out, dt, a.entries, a.O); CHECK_CONT(out);
  TORCH_CHECK(w.size(1) == (glu ? 2 : 1) * (int64_t)a.O && a.K % 64 == 0 &&
              (!glu || a.O % 64 == 0), "inner sizes must be padded");
  TORCH_CHECK((kind == 0) == (dt == at::kFloat), "kernels by dtype");
  a.out = out.data_ptr();
  a.x = x.data_ptr();
  a.w = w.data_ptr();
  a.ids = ids.data_ptr<int>();
  a.x_stride = x.stride(0);
  a.limit = (float)limit;
  a.alpha = (float)alpha;
  a.offset = (float)offset;
  a.cubic = (float)cubic;
  if (a.entries == 0) return;
  if (kind == 0) {
    TORCH_CHECK((a.O + 63) / 64 <= 65535, "grid");
    launch_experts_f32(glu, &a, cur_stream());
    return;
  }
  is_bf16(x);
  TORCH_CHECK(perm && offsets, "grouped entries");
  a.perm = opt_int(perm, a.entries);
  a.offsets = opt_int(offsets, a.E + 2);
  if (kind == 1) {
    TORCH_CHECK(tt == 1 || tt == 2, "token fragments");
    launch_experts_small(glu, &a, (int)tt, cur_stream());
    return;
  }
  TORCH_CHECK(tile_expert && a.K % 128 == 0, "tiles");
  a.tiles = a.entries / EXPERT_TILE + a.E;
  a.tile_expert = opt_int(tile_expert, a.tiles);
  a.tile_row = opt_int(tile_row, a.tiles);
  launch_experts_gemm(glu, &a, cur_stream());
}

static DeltaArgs delta_args(const torch::Tensor& out, const torch::Tensor& qkv,
                            const torch::Tensor& conv, const torch::Tensor& b,
                            const torch::Tensor& z, const torch::Tensor& A_log,
                            const torch::Tensor& dt_bias, const torch::Tensor& gate,
                            const torch::Tensor& norm, const torch::Tensor& state,
                            const torch::Tensor& ring, const torch::Tensor& seq_lens,
                            const torch::Tensor& slots, int64_t kv_heads, double eps,
                            double unit_eps, bool gate_silu) {
  const auto dt = qkv.scalar_type();
  DeltaArgs a{};
  CHECK_CUDA(state); CHECK_CONT(state);
  TORCH_CHECK(state.scalar_type() == at::kFloat && state.dim() == 4, "state layout");
  a.N = qkv.size(0);
  a.H = state.size(1);
  a.D = state.size(2);
  a.V = state.size(3);
  a.G = (int)kv_heads;
  TORCH_CHECK(a.G > 0 && a.H % a.G == 0 && a.D <= 1024 && a.V <= 1024, "delta rule: head sizes");
  a.C = 2 * a.G * a.D + a.H * a.V;
  a.taps = conv.size(1);
  check_rows(qkv, dt, a.N, a.C);
  check_rows(conv, dt, a.C, a.taps); CHECK_CONT(conv);
  check_rows(b, dt, a.N, a.H);
  a.head_decay = z.size(1) == a.H;
  const int64_t decays = (int64_t)a.H * (a.head_decay ? 1 : a.D);
  check_rows(z, dt, a.N, decays);
  check_rows(gate, dt, a.N, (int64_t)a.H * a.V);
  check_rows(out, dt, a.N, (int64_t)a.H * a.V); CHECK_CONT(out);
  check_vec(A_log, at::kFloat, a.H);
  check_vec(dt_bias, at::kFloat, decays);
  check_vec(norm, at::kFloat, a.V);
  CHECK_CUDA(ring); CHECK_CONT(ring);
  TORCH_CHECK(ring.scalar_type() == dt && ring.dim() == 3 && ring.size(0) == state.size(0) &&
              ring.size(1) == a.taps && ring.size(2) == a.C, "convolution state");
  is_bf16(qkv);
  a.seqs = seq_lens.numel();
  a.qkv = qkv.data_ptr();
  a.conv = conv.data_ptr();
  a.b = b.data_ptr();
  a.z = z.data_ptr();
  a.gate = gate.data_ptr();
  a.A_log = A_log.data_ptr<float>();
  a.dt_bias = dt_bias.data_ptr<float>();
  a.norm = norm.data_ptr<float>();
  a.state = state.data_ptr<float>();
  a.ring = ring.data_ptr();
  a.out = out.data_ptr();
  a.seq_lens = opt_int(seq_lens, a.seqs);
  a.slots = opt_int(slots, a.seqs);
  a.qkv_stride = qkv.stride(0);
  a.b_stride = b.stride(0);
  a.z_stride = z.stride(0);
  a.gate_stride = gate.stride(0);
  a.eps = (float)eps;
  a.unit_eps = (float)unit_eps;
  a.q_scale = 1.f / std::sqrt((float)a.D);
  a.gate_silu = gate_silu;
  return a;
}

// The rows of every chunk; y, unit, g, o: workspace (gated_delta.h)
static void delta_prompts(torch::Tensor out, torch::Tensor qkv, torch::Tensor conv,
                          torch::Tensor b, torch::Tensor z, torch::Tensor A_log,
                          torch::Tensor dt_bias, torch::Tensor gate, torch::Tensor norm,
                          torch::Tensor state, torch::Tensor ring, torch::Tensor seq_lens,
                          torch::Tensor slots, int64_t kv_heads, double eps, double unit_eps,
                          bool gate_silu, torch::Tensor ctx_lens, torch::Tensor row_starts,
                          torch::Tensor tile_seq, torch::Tensor tile_q0, torch::Tensor y,
                          torch::Tensor unit, OptTensor g, torch::Tensor o, int64_t cpl) {
  DeltaArgs a = delta_args(out, qkv, conv, b, z, A_log, dt_bias, gate, norm, state, ring,
                           seq_lens, slots, kv_heads, eps, unit_eps, gate_silu);
  check_vec(y, qkv.scalar_type(), (int64_t)a.N * a.C);
  check_vec(unit, at::kFloat, (int64_t)a.N * a.G * 3);
  if (!a.head_decay) {
    TORCH_CHECK(g, "workspace for the decays");
    check_vec(*g, at::kFloat, (int64_t)a.N * a.H * a.D);
    a.g = g->data_ptr<float>();
  }
  check_vec(o, at::kFloat, (int64_t)a.N * a.H * a.V);
  a.y = y.data_ptr();
  a.unit = unit.data_ptr<float>();
  a.o = o.data_ptr<float>();
  a.n_tiles = tile_seq.numel();
  a.ctx_lens = opt_int(ctx_lens, a.seqs);
  a.row_starts = opt_int(row_starts, a.seqs);
  a.tile_seq = opt_int(tile_seq, a.n_tiles);
  a.tile_q0 = opt_int(tile_q0, a.n_tiles);
  TORCH_CHECK(a.seqs <= 65535 && a.H <= 16384, "grid");
  if (a.N == 0 || a.n_tiles == 0) return;
  launch_delta_prompts(is_bf16(qkv), &a, (int)cpl, cur_stream());
}

// One token per sequence, row i of sequence i.
static void delta_step(torch::Tensor out, torch::Tensor qkv, torch::Tensor conv,
                       torch::Tensor b, torch::Tensor z, torch::Tensor A_log,
                       torch::Tensor dt_bias, torch::Tensor gate, torch::Tensor norm,
                       torch::Tensor state, torch::Tensor ring, torch::Tensor seq_lens,
                       torch::Tensor slots, int64_t kv_heads, double eps, double unit_eps,
                       bool gate_silu, int64_t threads) {
  DeltaArgs a = delta_args(out, qkv, conv, b, z, A_log, dt_bias, gate, norm, state, ring,
                           seq_lens, slots, kv_heads, eps, unit_eps, gate_silu);
  TORCH_CHECK(a.seqs == a.N && a.seqs <= 65535, "one token per sequence");
  TORCH_CHECK(threads % 64 == 0 && threads >= 64 && threads <= 1024 &&
              (a.V % 4 ? a.V : a.V / 4) <= threads, "threads");
  if (a.N == 0) return;
  launch_delta_step(is_bf16(qkv), &a, (int)threads, cur_stream());
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.doc() = "MI355X-native runtime: paged-KV block manager + CDNA4 kernels";
  register_block_manager(m);
  m.def("rmsnorm", &rmsnorm);
  m.def("fused_add_rmsnorm", &fused_add_rmsnorm);
  m.def("swiglu", &swiglu);
  m.def("rope_cache", &rope_cache);
  m.def("decode_attn", &decode_attn);
  m.def("prefill_attn", &prefill_attn);
  m.def("prefill_attn_mfma", &prefill_attn_mfma);
  m.def("mfma_probe", &mfma_probe);
  m.def("gemm_bf16", &gemm_bf16);
  m.attr("DEPTH_AHEAD") = DEPTH_AHEAD;
  m.def("residual_norm", &residual_norm);
  m.def("side_gate", &side_gate);
  m.def("add_to_residual", &add_to_residual);
  m.def("clamped_glu", &clamped_glu);
  m.def("gelu_gate", &gelu_gate);
  m.def("latent_inputs", &latent_inputs);
  m.def("head_linear", &head_linear);
  m.def("latent_attn", &latent_attn);
  m.def("latent_gather", &latent_gather);
  m.def("latent_prefill", &latent_prefill);
  m.def("embed_positions", &embed_positions);
  m.def("softcap", &softcap);
  m.def("cache_keys_values", &cache_keys_values);
  m.def("grouped_attn", &grouped_attn);
  m.def("talk_prefill_tokens", &talk_prefill_tokens);
  m.def("talk_decode_fits", &talk_decode_fits);
  m.def("attention_inputs", &attention_inputs);
  m.attr("EXPERT_TILE") = EXPERT_TILE;
  m.def("moe_route", &moe_route);
  m.def("moe_group", &moe_group);
  m.def("experts_linear", &experts_linear);
  m.def("delta_prompts", &delta_prompts);
  m.def("delta_step", &delta_step);
  m.def("sample", &sample);
  m.def("sample_fullvocab", &sample_fullvocab);
}
