// Shared by the bindings of the modules with latent attention (_latent, _latent_linear): the fp32 residual, the latent cache
// and the attention over it.
#pragma once
#include "bind_grouped.h"

extern "C" {
int pa_residual_norm(int fp32, float* resid, const void* y, int K, int ldy, float y_scale, const float* w_post,
                     const void* emb, const int* ids, int vocab, int emb_add, const float* mix, float* hist,
                     long long hist_step, int n_hist, const float* w_next, void* out, int ldo, const int* rows, int n, int D,
                     int post_groups, int next_groups, float eps, hipStream_t st);
int pa_latent_cache(int fp32, const void* x, int ldx, int NQ, int R, int r, int rd, const float* w_q, const float* w_c,
                    void* cq, int ldq, void* pages, int Rp, int D, const int* positions, const int* slots,
                    const float* cos_sin, float eps, int T, hipStream_t st);
int pa_latent_pad(int R);
int pa_latent_attention(int fp32, void* out, float* part_o, float* part_ml, const void* q, const void* pages,
                        const int* items, const int* n_items, int max_items, const int* q_start,
                        const int* q_len, const int* ctx_len, const int* block_table, int max_blocks, int H, int Rp,
                        int rp, int dec_tokens, int tile_tokens, int window, float scale_log2, int simple,
                        hipStream_t st);
}

namespace {

void residual_norm(at::Tensor resid, Opt y, int64_t K, double y_scale, Opt w_post, Opt emb, Opt ids, bool emb_add,
                   Opt w_next, Opt out, Opt rows, double eps, int64_t post_groups, int64_t next_groups, Opt mix, Opt hist) {
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
  TORCH_CHECK(!w_next.has_value() || out.has_value(), "w_next needs out");
  long long hist_step = 0;
  int n_hist = 0;
  if (mix.has_value()) {  // weights of the embedding, the earlier results and this one
    n_hist = mix->numel() - 1;
    TORCH_CHECK(hist.has_value() && emb.has_value() && n_hist >= 1, "a depth average needs hist and the embedding");
    check_gpu(*hist, "hist");
    check_dtype(*hist, at::kFloat, "hist");
    TORCH_CHECK(hist->dim() == 3 && hist->size(0) >= n_hist && hist->size(1) >= T && hist->size(2) == D, "hist must be [>= n, T, D]");
    hist_step = hist->stride(0);
  }
  if (out.has_value()) {
    check_rows(*out, dt, "out");
    TORCH_CHECK(out->size(0) >= n && out->size(1) >= D && out->stride(0) == out->size(1), "out must be [>= n, >= D]");
    ldo = out->stride(0);
  }
  check_rc(pa_residual_norm(dt == at::kFloat, resid.data_ptr<float>(), y.has_value() ? y->data_ptr() : nullptr, (int)K,
                            ldy, (float)y_scale, opt_f32(w_post, D, "w_post"), emb.has_value() ? emb->data_ptr() : nullptr,
                            emb.has_value() ? ints(*ids, T, "ids") : nullptr, emb.has_value() ? emb->size(0) : 0,
                            emb_add ? 1 : 0, opt_f32(mix, 2, "mix"), n_hist ? hist->data_ptr<float>() : nullptr, hist_step,
                            n_hist, opt_f32(w_next, D, "w_next"), out.has_value() ? out->data_ptr() : nullptr,
                            ldo, rows.has_value() ? ints(*rows, n, "rows") : nullptr, (int)n, (int)D, (int)post_groups,
                            (int)next_groups, (float)eps, cur_stream()),
           "residual_norm");
}

// x [T, NQ | R | r ..]; NQ 0: no query latent (w_q, cq null), r 0: no rotated part (cos_sin null)
void latent_cache(at::Tensor x, int64_t NQ, int64_t R, int64_t r, Opt w_q, at::Tensor w_c, Opt cq, at::Tensor pages,
                  int64_t Rp, at::Tensor positions, at::Tensor slots, Opt cos_sin, double eps) {
  const int f = is_f32(x, "x");
  check_rows(x, x.scalar_type(), "x");
  check_gpu(pages, "pages");
  check_dtype(pages, x.scalar_type(), "pages");
  TORCH_CHECK(pages.dim() == 4 && pages.size(2) == 16 && pages.size(3) == 8, "pages must be [blocks, D/8, 16, 8]");
  const int64_t T = x.size(0), D = pages.size(1) * 8;
  TORCH_CHECK(x.size(1) >= NQ + R + r && NQ >= 0 && R > 0 && r >= 0 && R <= Rp && Rp + r <= D, "latent_cache sizes");
  TORCH_CHECK(f || ((uintptr_t)x.data_ptr() & 15) == 0, "latent_cache: 16-byte aligned rows");
  TORCH_CHECK((NQ > 0) == cq.has_value() && (NQ > 0) == w_q.has_value() && (r > 0) == cos_sin.has_value(), "latent_cache parts");
  int64_t rd = 0;
  if (cos_sin.has_value()) {
    TORCH_CHECK(cos_sin->dim() == 2 && cos_sin->size(1) % 2 == 0 && cos_sin->size(1) <= r, "cos_sin must be [max_pos, dims <= r]");
    rd = cos_sin->size(1);
  }
  if (cq.has_value()) {
    check_rows(*cq, x.scalar_type(), "cq");
    TORCH_CHECK(cq->size(0) == T && cq->size(1) >= NQ && cq->stride(0) == cq->size(1), "cq must be [T, >= NQ]");
  }
  check_rc(pa_latent_cache(f, x.data_ptr(), x.stride(0), NQ, R, r, rd, opt_f32(w_q, NQ, "w_q"), opt_f32(w_c, R, "w_c"),
                           cq.has_value() ? cq->data_ptr() : nullptr, cq.has_value() ? cq->stride(0) : 0, pages.data_ptr(), Rp,
                           D, ints(positions, T, "positions"), ints(slots, T, "slots"), opt_f32(cos_sin, 0, "cos_sin"),
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
  TORCH_CHECK(Rp > 0 && rp >= 0 && dec_tokens >= 1 && tile_tokens >= 1, "latent_attention sizes");
  TORCH_CHECK(part_o.numel() >= mi * NB * 16 * Rp && part_ml.numel() >= mi * NB * 32, "partition workspace too small");
  check_rc(pa_latent_attention(f, out.data_ptr(), (float*)opt_f32(part_o, 0, "part_o"),
                               (float*)opt_f32(part_ml, 0, "part_ml"), q.data_ptr(),
                               pages.data_ptr(), ints(items, 0, "items"), ints(n_items, 1, "n_items"), mi,
                               ints(q_start, S, "q_start"), ints(q_len, S, "q_len"), ints(ctx_len, S, "ctx_len"),
                               ints(block_table, 0, "block_table"), block_table.size(1), H, Rp, rp, dec_tokens,
                               tile_tokens, window, (float)(scale * 1.4426950408889634), simple ? 1 : 0, cur_stream()),
           "latent_attention");
}

}  // namespace
