// Shared by the bindings of the modules with grouped projections (_latent, _hybrid, _latent_linear): operand checks and
// the per-head and sorted projections of grouped_gemm.hip.
#pragma once
#include "bind_common.h"

extern "C" {
int pa_grouped_gemm(int fp32, const void* x, const void* w, void* out, long long wstride, int groups, int ldx, int xg,
                    int ldo, int og, int rows, int N16, int K32, const int* tiles, int max_tiles, const int* n_tiles,
                    const int* order, int x_div, int out_order, int tm, int epi, float limit, float alpha, float cubic, float bias,
                    const int* positions, const float* cos_sin, int rskip, int r, int rp, int rd, const float* row_w,
                    const void* gate, int ldg, const void* table, const int* ids, int ldt, int tcol, int vocab, hipStream_t st);
}

namespace {

using Opt = c10::optional<at::Tensor>;

int is_f32(const at::Tensor& t, const char* name) {
  TORCH_CHECK(t.scalar_type() == at::kFloat || t.scalar_type() == at::kBFloat16, name, " must be bfloat16 or float32");
  return t.scalar_type() == at::kFloat ? 1 : 0;
}

// 2-D (rows x columns, unit inner stride) operand of the model's dtype
void check_rows(const at::Tensor& t, at::ScalarType dt, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.dim() == 2 && t.stride(1) == 1, name, " must be a 2-D GPU tensor, unit inner stride");
  check_dtype(t, dt, name);
}

const float* opt_f32(const Opt& t, int64_t n, const char* name) {
  if (!t.has_value()) return nullptr;
  check_gpu(*t, name);
  check_dtype(*t, at::kFloat, name);
  TORCH_CHECK(t->numel() >= n, name, " is too short");
  return t->data_ptr<float>();
}

const int* ints(const at::Tensor& t, int64_t n, const char* name) {
  check_gpu(t, name);
  check_dtype(t, at::kInt, name);
  TORCH_CHECK(t.numel() >= n, name, " is too short");
  return t.data_ptr<int>();
}

// w: bf16 packed [G, N/16, K/32, 64, 8] or fp32 [G, N, K]; epi 1: gated pair (out has N/2 columns per group)
void dims(const at::Tensor& w, int f, int64_t* G, int64_t* N, int64_t* K) {
  check_gpu(w, "w");
  if (f) {
    TORCH_CHECK(w.dim() == 3 && w.size(1) % 16 == 0 && w.size(2) % 32 == 0, "w must be [G, 16 n, 32 k]");
    *G = w.size(0); *N = w.size(1); *K = w.size(2);
  } else {
    TORCH_CHECK(w.dim() == 5 && w.size(3) == 64 && w.size(4) == 8, "w must be packed [G, N/16, K/32, 64, 8]");
    *G = w.size(0); *N = w.size(1) * 16; *K = w.size(2) * 32;
  }
}

// every row of x through every group: x columns g * xg .. + K -> out columns g * og .. + N; with
// positions / cos_sin also the rotated part: x columns g * xg + rskip .. + r -> out columns g * og + N .. + rp; with gate
// times sigmoid(gate), whose columns are out's
void head_gemm(at::Tensor x, int64_t xg, at::Tensor w, at::Tensor out, int64_t og, Opt positions, Opt cos_sin,
               int64_t rskip, int64_t r, int64_t rp, Opt gate) {
  const int f = is_f32(x, "x");
  check_rows(x, x.scalar_type(), "x");
  check_rows(out, x.scalar_type(), "out");
  check_dtype(w, x.scalar_type(), "w");
  int64_t G, N, K;
  dims(w, f, &G, &N, &K);
  TORCH_CHECK(out.size(0) == x.size(0) && (G - 1) * xg + K <= x.size(1) && (G - 1) * og + N <= out.size(1),
              "head_gemm sizes");
  const int* pos = nullptr;
  const float* cs = nullptr;
  int64_t rd = 0;
  if (positions.has_value()) {
    TORCH_CHECK(cos_sin.has_value() && cos_sin->dim() == 2 && cos_sin->size(1) % 2 == 0, "cos_sin must be [max_pos, dims]");
    rd = cos_sin->size(1);
    pos = ints(*positions, x.size(0), "positions");
    cs = opt_f32(cos_sin, 0, "cos_sin");
    TORCH_CHECK(rd <= r && r <= rp && rp > 0 && rskip >= 0 && (G - 1) * xg + rskip + r <= x.size(1) &&
                    (G - 1) * og + N + rp <= out.size(1), "head_gemm rotation sizes");
  } else {
    rp = 0;
  }
  if (gate.has_value()) {
    check_rows(*gate, x.scalar_type(), "gate");
    TORCH_CHECK(gate->size(0) == x.size(0) && gate->size(1) >= (G - 1) * og + N && gate->stride(0) % 4 == 0 &&
                    ((uintptr_t)gate->data_ptr() & 7) == 0, "head_gemm: gate must be [rows, >= out's columns]");
  }
  TORCH_CHECK(f || (x.stride(0) % 8 == 0 && xg % 8 == 0 && out.stride(0) % 4 == 0 && og % 4 == 0),
              "head_gemm: 16-byte aligned operands");
  check_rc(pa_grouped_gemm(f, x.data_ptr(), w.data_ptr(), out.data_ptr(), N * K, G, x.stride(0), xg, out.stride(0), og,
                           x.size(0), N / 16, K / 32, nullptr, 0, nullptr, nullptr, 0, 0, 0, gate.has_value() ? 3 : 0, 0.f, 0.f,
                           0.f, 0.f, pos, cs, rskip, r, rp, rd, nullptr, gate.has_value() ? gate->data_ptr() : nullptr,
                           gate.has_value() ? gate->stride(0) : 0, nullptr, nullptr, 0, 0, 0, cur_stream()),
           "head_gemm");
}

// out = gated unit of (x w^T, the row's embedding): table [vocab, columns], from column tcol on
void table_gemm(at::Tensor x, at::Tensor w, at::Tensor out, at::Tensor table, at::Tensor ids, int64_t tcol, double limit,
                double alpha, double bias, double cubic) {
  const int f = is_f32(x, "x");
  for (auto* t : {&x, &out, &table}) check_rows(*t, x.scalar_type(), "table_gemm operand");
  check_dtype(w, x.scalar_type(), "w");
  int64_t G, N, K;
  dims(w, f, &G, &N, &K);
  TORCH_CHECK(G == 1 && out.size(0) == x.size(0) && K <= x.size(1) && N <= out.size(1) && tcol >= 0 &&
                  tcol + N <= table.size(1) && table.size(0) > 0, "table_gemm sizes");
  TORCH_CHECK(f || (x.stride(0) % 8 == 0 && out.stride(0) % 4 == 0 && table.stride(0) % 4 == 0 && tcol % 4 == 0 &&
                    ((uintptr_t)x.data_ptr() & 15) == 0 && ((uintptr_t)out.data_ptr() & 7) == 0),
              "table_gemm: 16-byte aligned operands");
  check_rc(pa_grouped_gemm(f, x.data_ptr(), w.data_ptr(), out.data_ptr(), N * K, 1, x.stride(0), 0, out.stride(0), 0,
                           x.size(0), N / 16, K / 32, nullptr, 0, nullptr, nullptr, 0, 0, 0, 4, (float)limit, (float)alpha,
                           (float)cubic, (float)bias, nullptr, nullptr, 0, 0, 0, 0, nullptr, nullptr, 0, table.data_ptr(),
                           ints(ids, x.size(0), "ids"), table.stride(0), (int)tcol, table.size(0), cur_stream()),
           "table_gemm");
}

// rows sorted by group: x row = order[p] / x_div (x_div 0: p), out row = out_order ? order[p] : p; epi 1: the gated
// unit, 2: the square of relu; row_w: weights of x's rows by order[p] (epi 1)
void expert_gemm(at::Tensor x, at::Tensor w, at::Tensor out, at::Tensor tiles, at::Tensor n_tiles, at::Tensor order,
                 int64_t rows, int64_t x_div, bool out_order, int64_t tm, int64_t epi, double limit, double alpha,
                 double bias, double cubic, Opt row_w) {
  const int f = is_f32(x, "x");
  check_rows(x, x.scalar_type(), "x");
  check_rows(out, x.scalar_type(), "out");
  check_dtype(w, x.scalar_type(), "w");
  int64_t G, N, K;
  dims(w, f, &G, &N, &K);
  TORCH_CHECK(K <= x.size(1) && epi >= 0 && epi <= 2 && (epi == 1 ? N / 2 : N) <= out.size(1) && out.size(0) >= rows &&
                  x.size(0) * (x_div ? x_div : 1) >= rows, "expert_gemm sizes");
  TORCH_CHECK(f || (x.stride(0) % 8 == 0 && out.stride(0) % 4 == 0 && ((uintptr_t)out.data_ptr() & 7) == 0),
              "expert_gemm: 16-byte aligned rows");
  TORCH_CHECK(tm != 256 || (!f && K % 64 == 0 && K >= 128 && N % 128 == 0 && out.stride(0) % 8 == 0 &&
                               ((uintptr_t)out.data_ptr() & 15) == 0),
              "expert_gemm: tiles of 256 rows need K % 64 == 0, K >= 128, N % 128 == 0");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 4, "tiles must be [n, 4]");
  check_rc(pa_grouped_gemm(f, x.data_ptr(), w.data_ptr(), out.data_ptr(), N * K, G, x.stride(0), 0, out.stride(0), 0, 0,
                           N / 16, K / 32, ints(tiles, 4, "tiles"), tiles.size(0), ints(n_tiles, 1, "n_tiles"),
                           ints(order, rows, "order"), x_div, out_order ? 1 : 0, tm, (int)epi, (float)limit,
                           (float)alpha, (float)cubic, (float)bias, nullptr, nullptr, 0, 0, 0, 0, opt_f32(row_w, rows, "row_w"),
                           nullptr, 0, nullptr, nullptr, 0, 0, 0, cur_stream()),
           "expert_gemm");
}

}  // namespace
