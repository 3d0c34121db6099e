// Python bindings of the latent-attention / expert-table kernels (module _latent): the kernels a
// model with an fp32 residual stream, latent attention and table-routed experts runs, beside the
// packed-weight projections it shares with the other models. Built as its own module so that such
// a model needs no other kernel. Every entry point checks shapes on the host and launches on the
// caller's stream.
#include "bind_grouped.h"

extern "C" {
int pa_residual_norm(int fp32, float* resid, const void* y, int K, int ldy, float y_scale, const float* w_post,
                     const void* emb, const int* ids, int vocab, int emb_add, const float* w_next, void* out, int ldo,
                     const int* rows, int n, int D, float eps, hipStream_t st);
int pa_latent_cache(int fp32, const void* x, int ldx, int NQ, int R, int r, int rd, const float* w_q, const float* w_c,
                    void* cq, int ldq, void* pages, int Rp, int D, const int* positions, const int* slots,
                    const float* cos_sin, float eps, int T, hipStream_t st);
int pa_latent_pad(int R);
int pa_latent_attention(int fp32, void* out, float* part_o, float* part_ml, const void* q, const void* pages,
                        const int* items, const int* n_items, int max_items, const int* q_start,
                        const int* q_len, const int* ctx_len, const int* block_table, int max_blocks, int H, int Rp,
                        int rp, int dec_tokens, int tile_tokens, int window, float scale_log2, int simple,
                        hipStream_t st);
int pa_table_route(const int* tables, const int* desc, int layers, const int* ids, const int* slots, int T, int tm,
                   int* order, int* tiles, int* n_tiles, hipStream_t st);
}

namespace {

void residual_norm(at::Tensor resid, Opt y, int64_t K, double y_scale, Opt w_post, Opt emb, Opt ids, bool emb_add,
                   Opt w_next, Opt out, Opt rows, double eps) {
  check_gpu(resid, "resid");
  check_dtype(resid, at::kFloat, "resid");
  TORCH_CHECK(resid.dim() == 2, "resid must be [T, D]");
  const int64_t T = resid.size(0), D = resid.size(1), n = rows.has_value() ? rows->numel() : T;
  at::ScalarType dt = at::kFloat;
  for (const Opt* o : {&y, &emb, &out})
    if (o->has_value()) dt = (*o)->scalar_type();
  int ldy = 0, ldo = 0;
  if (y.has_value()) {
    check_rows(*y, dt, "y");
    TORCH_CHECK(K >= 1 && y->size(0) == T * K && y->size(1) >= D, "y must be [T * K, >= D]");
    ldy = y->stride(0);
  }
  if (emb.has_value()) {
    check_gpu(*emb, "emb");
    check_dtype(*emb, dt, "emb");
    TORCH_CHECK(ids.has_value() && emb->dim() == 2 && emb->size(1) == D && emb->size(0) > 0, "emb must be [vocab, D]");
  }
  TORCH_CHECK(w_next.has_value() == out.has_value(), "w_next and out go together");
  if (out.has_value()) {
    check_rows(*out, dt, "out");
    TORCH_CHECK(out->size(0) >= n && out->size(1) >= D && out->stride(0) == out->size(1), "out must be [>= n, >= D]");
    ldo = out->stride(0);
  }
  check_rc(pa_residual_norm(dt == at::kFloat, resid.data_ptr<float>(), y.has_value() ? y->data_ptr() : nullptr, (int)K,
                            ldy, (float)y_scale, opt_f32(w_post, D, "w_post"), emb.has_value() ? emb->data_ptr() : nullptr,
                            emb.has_value() ? ints(*ids, T, "ids") : nullptr, emb.has_value() ? emb->size(0) : 0,
                            emb_add ? 1 : 0, opt_f32(w_next, D, "w_next"), out.has_value() ? out->data_ptr() : nullptr,
                            ldo, rows.has_value() ? ints(*rows, n, "rows") : nullptr, (int)n, (int)D, (float)eps,
                            cur_stream()),
           "residual_norm");
}

void latent_cache(at::Tensor x, int64_t NQ, int64_t R, int64_t r, at::Tensor w_q, at::Tensor w_c, at::Tensor cq,
                  at::Tensor pages, int64_t Rp, at::Tensor positions, at::Tensor slots, at::Tensor cos_sin,
                  double eps) {
  const int f = is_f32(x, "x");
  check_rows(x, x.scalar_type(), "x");
  check_rows(cq, x.scalar_type(), "cq");
  check_gpu(pages, "pages");
  check_dtype(pages, x.scalar_type(), "pages");
  TORCH_CHECK(pages.dim() == 4 && pages.size(2) == 16 && pages.size(3) == 8, "pages must be [blocks, D/8, 16, 8]");
  const int64_t T = x.size(0), D = pages.size(1) * 8;
  check_gpu(cos_sin, "cos_sin");
  check_dtype(cos_sin, at::kFloat, "cos_sin");
  TORCH_CHECK(cos_sin.dim() == 2 && cos_sin.size(1) % 2 == 0 && cos_sin.size(1) <= r, "cos_sin must be [max_pos, dims <= r]");
  TORCH_CHECK(x.size(1) >= NQ + R + r && NQ > 0 && R > 0 && R <= Rp && Rp + r <= D, "latent_cache sizes");
  TORCH_CHECK(cq.size(0) == T && cq.size(1) >= NQ && cq.stride(0) == cq.size(1), "cq must be [T, >= NQ]");
  check_rc(pa_latent_cache(f, x.data_ptr(), x.stride(0), NQ, R, r, cos_sin.size(1), opt_f32(w_q, NQ, "w_q"),
                           opt_f32(w_c, R, "w_c"), cq.data_ptr(), cq.stride(0), pages.data_ptr(), Rp, D,
                           ints(positions, T, "positions"), ints(slots, T, "slots"), cos_sin.data_ptr<float>(),
                           (float)eps, T, cur_stream()),
           "latent_cache");
}

void latent_attention(at::Tensor out, at::Tensor part_o, at::Tensor part_ml, at::Tensor q,
                      at::Tensor pages, at::Tensor items, at::Tensor n_items, at::Tensor q_start, at::Tensor q_len,
                      at::Tensor ctx_len, at::Tensor block_table, int64_t dec_tokens, int64_t tile_tokens,
                      int64_t window, double scale, bool simple) {
  const int f = is_f32(q, "q");
  for (auto* t : {&out, &q, &pages}) {
    check_gpu(*t, "latent_attention arg");
    check_dtype(*t, q.scalar_type(), "latent_attention arg");
  }
  TORCH_CHECK(q.dim() == 3 && out.dim() == 3 && out.size(0) == q.size(0) && out.size(1) == q.size(1),
              "q [T, H, D], out [T, H, Rp]");
  TORCH_CHECK(pages.dim() == 4 && pages.size(1) * 8 == q.size(2) && pages.size(2) == 16 && pages.size(3) == 8,
              "pages must be [blocks, D/8, 16, 8]");
  TORCH_CHECK(items.dim() == 2 && items.size(1) == 4 && block_table.dim() == 2, "items [n, 4], block_table [seqs, blocks]");
  const int64_t H = q.size(1), Rp = out.size(2), rp = q.size(2) - Rp, S = block_table.size(0), mi = items.size(0);
  const int64_t NB = (dec_tokens * H + 15) / 16;
  TORCH_CHECK(Rp > 0 && rp > 0 && dec_tokens >= 1 && tile_tokens >= 1, "latent_attention sizes");
  TORCH_CHECK(part_o.numel() >= mi * NB * 16 * Rp && part_ml.numel() >= mi * NB * 32, "partition workspace too small");
  check_rc(pa_latent_attention(f, out.data_ptr(), (float*)opt_f32(part_o, 0, "part_o"),
                               (float*)opt_f32(part_ml, 0, "part_ml"), q.data_ptr(),
                               pages.data_ptr(), ints(items, 0, "items"), ints(n_items, 1, "n_items"), mi,
                               ints(q_start, S, "q_start"), ints(q_len, S, "q_len"), ints(ctx_len, S, "ctx_len"),
                               ints(block_table, 0, "block_table"), block_table.size(1), H, Rp, rp, dec_tokens,
                               tile_tokens, window, (float)(scale * 1.4426950408889634), simple ? 1 : 0, cur_stream()),
           "latent_attention");
}

// desc [layers, 8]: table offset, vocab, top, experts, order offset, tile offset, max tiles, 0 (host copy checked)
void table_route(at::Tensor tables, at::Tensor desc, at::Tensor desc_host, at::Tensor ids, at::Tensor slots, int64_t T,
                 int64_t tm, at::Tensor order, at::Tensor tiles, at::Tensor n_tiles) {
  TORCH_CHECK(desc_host.device().is_cpu() && desc_host.dtype() == at::kInt && desc_host.dim() == 2 &&
                  desc_host.size(1) == 8 && desc_host.is_contiguous(), "desc_host must be int32 [layers, 8] on the CPU");
  const int64_t L = desc_host.size(0);
  const int* d = desc_host.data_ptr<int>();
  for (int64_t l = 0; l < L; ++l, d += 8)
    TORCH_CHECK(d[3] >= 1 && d[3] <= 2048 && d[2] >= 1 && d[0] >= 0 && (int64_t)d[0] + (int64_t)d[1] * d[2] <= tables.numel() &&
                    d[4] >= 0 && d[4] + T * d[2] <= order.numel() && d[5] >= 0 &&
                    ((int64_t)d[5] + d[6]) * 4 <= tiles.numel() && tm >= 1,
                "table_route: layer ", l, " does not fit its buffers");
  check_rc(pa_table_route(ints(tables, 1, "tables"), ints(desc, L * 8, "desc"), L, ints(ids, T, "ids"),
                          ints(slots, T, "slots"), T, tm, (int*)ints(order, 0, "order"), (int*)ints(tiles, 0, "tiles"),
                          (int*)ints(n_tiles, L, "n_tiles"), cur_stream()),
           "table_route");
}

}  // namespace

PYBIND11_MODULE(_latent, m) {
  m.doc() = "pilottai_amd CDNA4 (gfx950) kernels: latent attention, table-routed experts, fp32 residual";
  m.def("residual_norm", &residual_norm);
  m.def("latent_cache", &latent_cache);
  m.def("latent_pad", [](int R) { return pa_latent_pad(R); });
  m.def("latent_attention", &latent_attention);
  m.def("table_route", &table_route);
  m.def("head_gemm", &head_gemm);
  m.def("expert_gemm", &expert_gemm);
  m.def("empty_uncached", &empty_uncached);
  m.def("decode_gemm", &decode_gemm);
  m.def("prefill_gemm", &prefill_gemm);
}
