// Shared by the bindings of the modules with recurrent layers and score-routed experts (_hybrid, _latent_linear): the gated
// norm behind a recurrence and the routing.
#pragma once
#include "bind_grouped.h"

extern "C" {
int pa_gated_norm(int fp32, void* y, int ldy, int cols, const void* z, int ldz, const float* w, const int* slots,
                  const float* div, int after, int T, int H, int V, int Vp, int parts, float eps, hipStream_t st);
int pa_score_route(int fp32, const void* h, int ldh, const void* w, int K, const int* slots, float* weights,
                   int* choice, int* rank, int* counts, int* order, int* tiles, int* n_tiles, int T, int E, int top,
                   int groups, int keep, int always, int tm, int max_tiles, int softmax, const float* correction, int share,
                   float scale, hipStream_t st);
}

namespace {

int* out_ints(const at::Tensor& t, int64_t n, const char* name) { return const_cast<int*>(ints(t, n, name)); }

void gated_norm(at::Tensor y, at::Tensor z, at::Tensor w, at::Tensor slots, int64_t H, int64_t V, int64_t Vp,
                int64_t parts, double eps, Opt div, int64_t after) {
  const int f = is_f32(y, "y");
  check_rows(y, y.scalar_type(), "y");
  check_rows(z, y.scalar_type(), "z");
  const int64_t T = y.size(0);
  TORCH_CHECK(z.size(0) == T && y.size(1) >= H * Vp && z.size(1) >= H * Vp && V <= Vp && parts > 0 && after >= 0 && after <= 2, "gated_norm sizes");
  check_rc(pa_gated_norm(f, y.data_ptr(), y.stride(0), y.size(1), z.data_ptr(), z.stride(0), opt_f32(w, H * V, "w"),
                         ints(slots, T, "slots"), opt_f32(div, T * H, "div"), (int)after, T, H, V, Vp, parts, (float)eps,
                         cur_stream()),
           "gated_norm");
}

void score_route(at::Tensor h, at::Tensor w, at::Tensor slots, at::Tensor weights, at::Tensor choice, at::Tensor rank,
                 at::Tensor counts, at::Tensor order, at::Tensor tiles, at::Tensor n_tiles, int64_t E, int64_t top,
                 int64_t groups, int64_t keep, int64_t always, int64_t tm, bool softmax, Opt correction, bool share,
                 double scale) {
  const int f = is_f32(h, "h");
  check_rows(h, h.scalar_type(), "h");
  check_dtype(w, h.scalar_type(), "w");
  int64_t G, N, K;
  dims(w, f, &G, &N, &K);
  const int64_t T = h.size(0), P = T * (top + always);
  TORCH_CHECK(G == 1 && N >= E && K <= h.size(1) && h.stride(0) % 8 == 0 && tm >= 1, "score_route sizes");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 4, "tiles must be [n, 4]");
  check_rc(pa_score_route(f, h.data_ptr(), h.stride(0), w.data_ptr(), K, ints(slots, T, "slots"),
                          (float*)opt_f32(weights, P, "weights"), out_ints(choice, P, "choice"), out_ints(rank, P, "rank"),
                          out_ints(counts, E + always, "counts"), out_ints(order, P, "order"), out_ints(tiles, 4, "tiles"),
                          out_ints(n_tiles, 1, "n_tiles"), T, E, top, groups, keep, always, tm, tiles.size(0), softmax ? 1 : 0,
                          opt_f32(correction, E, "correction"), share ? 1 : 0, (float)scale, cur_stream()),
           "score_route");
}

}  // namespace
