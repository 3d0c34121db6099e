// Python bindings of the kernels of models that mix latent attention with gated linear attention (module
// _latent_linear): both, the fp32 residual with group norms and depth averages, score-routed experts and polynomial
// norms, beside the packed-weight and grouped projections they share with the other models. Built as its own module
// so that such a model needs no other kernel. Every entry point checks shapes on the host and launches on the caller's
// stream.
#include "bind_latent.h"
#include "bind_mixed.h"

extern "C" {
int pa_linear_attention(int fp32, const void* x, int ldx, void* y, int ldy, float* state, float* work, void* qd, void* kd,
                        void* sc, float* end, const void* a2, const float* bias, const int* q_start, const int* q_len,
                        const int* ctx_len, const int* state_slot, const int* items, const int* n_items, int max_items,
                        int seqs, int T, int H, int V, int N, int rp, int cq, int ck, int cv, int ca, float q_scale,
                        float inv_tau, int scan_min, hipStream_t st);
int pa_poly_norm(int fp32, void* z, int ld, int rows, int n, int cols, const float* act, float eps, hipStream_t st);
}

namespace {

// cols: where q, k, v and the low-rank inputs of the decays start; room: q', k' and scores of `max_items` > 0 chunks
void linear_attention(at::Tensor x, at::Tensor y, at::Tensor state, at::Tensor work, at::Tensor qd, at::Tensor kd, at::Tensor sc,
                      at::Tensor end, at::Tensor a2, at::Tensor bias, at::Tensor q_start, at::Tensor q_len, at::Tensor ctx_len,
                      at::Tensor state_slot, at::Tensor items, at::Tensor n_items, int64_t max_items, int64_t seqs,
                      std::vector<int64_t> cols, double q_scale, double inv_tau, int64_t scan_min) {
  const int f = is_f32(x, "x");
  check_rows(x, x.scalar_type(), "x");
  check_rows(y, x.scalar_type(), "y");
  for (auto* t : {&state, &work, &end, &bias}) {
    check_gpu(*t, "a state");
    check_dtype(*t, at::kFloat, "a state");
  }
  for (auto* t : {&qd, &kd, &sc, &a2}) {
    check_gpu(*t, "linear_attention operand");
    check_dtype(*t, x.scalar_type(), "linear_attention operand");
  }
  TORCH_CHECK(state.dim() == 4 && a2.dim() == 2 && cols.size() == 4, "state [slots, H, V, N], a2 [H N, rank], cols: q, k, v, a");
  const int64_t T = x.size(0), H = state.size(1), V = state.size(2), N = state.size(3), rp = a2.size(1), C = x.size(1);
  TORCH_CHECK(a2.size(0) == H * N && bias.numel() == H * N, "a2 and bias must have H N rows");
  TORCH_CHECK(cols[0] >= 0 && cols[0] + H * N <= C && cols[1] >= 0 && cols[1] + H * N <= C && cols[2] >= 0 &&
                  cols[2] + H * V <= C && cols[3] >= 0 && cols[3] + rp <= C, "x has too few columns");
  TORCH_CHECK(y.size(0) == T && y.size(1) >= H * V, "y must be [T, >= H * V]");
  TORCH_CHECK(((uintptr_t)x.data_ptr() & 15) == 0 && ((uintptr_t)y.data_ptr() & 7) == 0, "16-byte aligned rows");
  TORCH_CHECK(seqs <= q_start.numel() && items.numel() >= 4 * max_items, "linear_attention: sequences and items");
  if (!f && max_items > 0)
    TORCH_CHECK(work.numel() >= max_items * H * V * N && end.numel() >= max_items * H * N && qd.numel() >= 2 * T * H * N &&
                    kd.numel() >= 2 * T * H * N && sc.numel() >= 2 * T * H * 64, "linear_attention: workspace too small");
  check_rc(pa_linear_attention(f, x.data_ptr(), x.stride(0), y.data_ptr(), y.stride(0), state.data_ptr<float>(),
                               work.data_ptr<float>(), qd.data_ptr(), kd.data_ptr(), sc.data_ptr(), end.data_ptr<float>(),
                               a2.data_ptr(), bias.data_ptr<float>(), ints(q_start, seqs, "q_start"), ints(q_len, seqs, "q_len"),
                               ints(ctx_len, seqs, "ctx_len"), ints(state_slot, seqs, "state_slot"), ints(items, 0, "items"),
                               ints(n_items, 1, "n_items"), max_items, seqs, T, H, V, N, rp, cols[0], cols[1], cols[2], cols[3],
                               (float)q_scale, (float)inv_tau, scan_min, cur_stream()),
           "linear_attention");
}

void poly_norm(at::Tensor z, int64_t n, at::Tensor act, double eps) {
  check_rows(z, z.scalar_type(), "z");
  TORCH_CHECK(n >= 1 && n <= z.size(1), "poly_norm sizes");
  check_rc(pa_poly_norm(is_f32(z, "z"), z.data_ptr(), z.stride(0), z.size(0), n, z.size(1), opt_f32(act, 4, "act"), (float)eps,
                        cur_stream()),
           "poly_norm");
}

}  // namespace

PYBIND11_MODULE(_latent_linear, m) {
  m.doc() = "pilottai_amd CDNA4 (gfx950) kernels: latent and gated linear attention, depth averages, score-routed experts";
  m.def("residual_norm", &residual_norm);
  m.def("latent_cache", &latent_cache);
  m.def("latent_pad", [](int R) { return pa_latent_pad(R); });
  m.def("latent_attention", &latent_attention);
  m.def("linear_attention", &linear_attention);
  m.def("gated_norm", &gated_norm);
  m.def("poly_norm", &poly_norm);
  m.def("score_route", &score_route);
  m.def("head_gemm", &head_gemm);
  m.def("table_gemm", &table_gemm);
  m.def("expert_gemm", &expert_gemm);
  m.def("empty_uncached", &empty_uncached);
  m.def("decode_gemm", &decode_gemm);
  m.def("prefill_gemm", &prefill_gemm);
}
