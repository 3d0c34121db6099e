// Python bindings of the kernels of hybrid models (module _hybrid): attention over paged keys and values with its masks,
// biases and gates, state-space and matrix-memory layers, score-routed experts and fp32 residuals, beside the
// packed-weight and grouped projections they share with the other models. Built as its own module so that such a
// model needs no other kernel. Every entry point checks shapes on the host and launches on the caller's
// stream.
#include "bind_mixed.h"

extern "C" {
int pa_hyper_norm(int fp32, float* x, int S, const void* y, int K, int ldy, const float* y_w, const void* y2, int ldy2,
                  const float* bias, const float* mix, const float* post, const float* pre, const void* emb, const int* ids, int vocab,
                  const float* w_next, void* out, int ldo, const int* rows, int n, int D, float eps, hipStream_t st);
int pa_softcap(int fp32, void* x, int ld, int rows, int cols, float cap, hipStream_t st);
int pa_paged_kv(int fp32, const void* x, const float* bias, void* q, void* kp, void* vp, void* pk, void* pv,
                const int* positions, const int* slots, const int* q_start, const int* q_len, const int* ctx_len,
                const int* block_table, const float* cos_sin, int ldx, int H, int G, int GV, int DK, int DV, int rd, int pool,
                int npb, int max_blocks, int max_seqs, int T, int vcol, const float* qn, const float* kn, int norm_v, int dim,
                int vdim, float eps, hipStream_t st);
void pa_window_pad(int k, int v, int* dk, int* dv);
int pa_window_attention(int fp32, void* out, int out_f32, int ldo, float* part_o, float* part_ml, const void* q,
                        const void* kp, const void* vp, const void* pk, const void* pv, const int* items, const int* n_items,
                        int max_items, const int* q_start, const int* q_len, const int* ctx_len, const int* block_table,
                        int max_blocks, int T, int H, int G, int GV, int DK, int DV, int dec_tokens, int tile_tokens,
                        int window, int pool, int npb, int keep, int chunk, int max_slots, float scale, const float* slopes,
                        float cap, const float* sink, const void* gate, int ldg, float gain, int simple, hipStream_t st);
int pa_head_difference(int fp32, const float* a, void* out, int ldo, const void* gate, int ldg, int T, int H, int groups, int D,
                       float lam, float gain, int vdim, float eps, hipStream_t st);
int pa_matrix_memory(int fp32, const void* x, int ldx, void* y, int ldy, float* div, float* state, float* top, float* work,
                     float* stat, const float* i_bias, const float* f_bias, const int* q_start, const int* q_len,
                     const int* ctx_len, const int* state_slot, const int* items, const int* n_items, int max_items, int seqs,
                     int H, int V, int N, int cq, int ck, int cv, int ci, int vin, int vdim, float cap, float q_scale,
                     int scan_min, hipStream_t st);
int pa_state_scan(int fp32, const void* proj, int ldp, void* u, void* y, int ldy, float* state, void* ring, float* work,
                  float* total, const float* conv_w, const float* conv_b, const float* dt_bias, const float* a,
                  const float* d, const int* q_start, const int* q_len, const int* ctx_len, const int* state_slot,
                  const int* scan_first, const int* items, const int* n_items, int max_items, int seqs, int H, int G,
                  int V, int N, int taps, int ring_rows, int scan_min, hipStream_t st);
}

namespace {

// a step's sequences: q_start, q_len, ctx_len [S], block_table [S, blocks]
int64_t seqs_of(const at::Tensor& block_table) {
  TORCH_CHECK(block_table.dim() == 2, "block_table must be [seqs, blocks]");
  return block_table.size(0);
}

void hyper_norm(at::Tensor x, Opt y, int64_t K, Opt y_w, Opt y2, Opt bias, Opt mix, Opt post, Opt pre, Opt emb, Opt ids,
                Opt w_next, Opt out, Opt rows, double eps) {
  check_gpu(x, "x");
  check_dtype(x, at::kFloat, "x");
  TORCH_CHECK(x.dim() == 3, "x must be [T, streams, D]");
  const int64_t T = x.size(0), S = x.size(1), D = x.size(2), n = rows.has_value() ? rows->numel() : T;
  at::ScalarType dt = at::kFloat;
  for (const Opt* o : {&y, &emb, &out})
    if (o->has_value()) dt = (*o)->scalar_type();
  int ldy = 0, ldy2 = 0, ldo = 0;
  if (y.has_value()) {
    check_rows(*y, dt, "y");
    TORCH_CHECK(K >= 1 && y->size(0) == T * K && y->size(1) >= D && mix.has_value() && post.has_value(),
                "y must be [T * K, >= D], with mix and post");
    ldy = y->stride(0);
  }
  if (y2.has_value()) {
    check_rows(*y2, dt, "y2");
    TORCH_CHECK(y.has_value() && y2->size(0) == T && y2->size(1) >= D, "y2 must be [T, >= D], beside y");
    ldy2 = y2->stride(0);
  }
  if (emb.has_value()) {
    check_gpu(*emb, "emb");
    check_dtype(*emb, dt, "emb");
    TORCH_CHECK(ids.has_value() && emb->dim() == 2 && emb->size(1) == D && emb->size(0) > 0, "emb must be [vocab, D]");
  }
  TORCH_CHECK(w_next.has_value() == out.has_value() && (!out.has_value() || pre.has_value()), "w_next, pre and out go together");
  if (out.has_value()) {
    check_rows(*out, dt, "out");
    TORCH_CHECK(out->size(0) >= n && out->size(1) >= D && out->stride(0) == out->size(1), "out must be [>= n, >= D]");
    ldo = out->stride(0);
  }
  check_rc(pa_hyper_norm(dt == at::kFloat, x.data_ptr<float>(), S, y.has_value() ? y->data_ptr() : nullptr, (int)K, ldy,
                         opt_f32(y_w, T * K, "y_w"), y2.has_value() ? y2->data_ptr() : nullptr, ldy2, opt_f32(bias, D, "bias"), opt_f32(mix, S * S, "mix"),
                         opt_f32(post, S, "post"), opt_f32(pre, S, "pre"), emb.has_value() ? emb->data_ptr() : nullptr,
                         emb.has_value() ? ints(*ids, T, "ids") : nullptr, emb.has_value() ? emb->size(0) : 0,
                         opt_f32(w_next, D, "w_next"), out.has_value() ? out->data_ptr() : nullptr, ldo,
                         rows.has_value() ? ints(*rows, n, "rows") : nullptr, (int)n, (int)D, (float)eps, cur_stream()),
           "hyper_norm");
}

void softcap(at::Tensor x, int64_t cols, double cap) {
  check_rows(x, x.scalar_type(), "x");
  TORCH_CHECK(cols <= x.size(1) && cap > 0, "softcap sizes");
  check_rc(pa_softcap(is_f32(x, "x"), x.data_ptr(), x.stride(0), x.size(0), cols, (float)cap, cur_stream()), "softcap");
}

struct Pools {
  int64_t G, GV, DK, DV, npb;
};

Pools check_pools(const at::Tensor& kp, const at::Tensor& vp, const at::Tensor& pk, const at::Tensor& pv,
                  at::ScalarType dt, int64_t pool) {
  for (auto* t : {&kp, &vp, &pk, &pv}) {
    check_gpu(*t, "cache pool");
    check_dtype(*t, dt, "cache pool");
  }
  TORCH_CHECK(kp.dim() == 5 && vp.dim() == 5 && kp.size(3) == 16 && kp.size(4) == 8 && vp.size(3) == 16 &&
                  vp.size(4) == 8 && kp.size(0) == vp.size(0) && kp.size(1) % vp.size(1) == 0,
              "pages must be [blocks, G, D/8, 16, 8]");
  const Pools p{kp.size(1), vp.size(1), kp.size(2) * 8, vp.size(2) * 8, pool > 0 ? pk.size(1) : 1};
  if (pool > 0)
    TORCH_CHECK(p.G == p.GV && pk.dim() == 4 && pv.dim() == 4 && pk.size(0) == kp.size(0) && pv.size(0) == kp.size(0) &&
                    pv.size(1) == p.npb && p.npb * pool >= 16 && pk.size(2) == p.G && pv.size(2) == p.G &&
                    pk.size(3) == p.DK && pv.size(3) == p.DV, "pooled rows must be [blocks, per page, G, D]");
  return p;
}

void paged_kv(at::Tensor x, Opt bias, at::Tensor q, at::Tensor kp, at::Tensor vp, at::Tensor pk, at::Tensor pv,
              at::Tensor positions, at::Tensor slots, at::Tensor q_start, at::Tensor q_len, at::Tensor ctx_len,
              at::Tensor block_table, Opt cos_sin, int64_t pool, int64_t v_col, Opt q_norm, Opt k_norm, bool norm_v,
              int64_t dim, int64_t vdim, double eps) {
  const int f = is_f32(x, "x");
  check_rows(x, x.scalar_type(), "x");
  check_gpu(q, "q");
  check_dtype(q, x.scalar_type(), "q");
  const Pools p = check_pools(kp, vp, pk, pv, x.scalar_type(), pool);
  const int64_t T = x.size(0), S = seqs_of(block_table);
  TORCH_CHECK(q.dim() == 3 && q.size(0) == T && q.size(2) == p.DK, "q must be [T, H, DK]");
  const int64_t H = q.size(1), vcol = v_col < 0 ? (H + p.G) * p.DK : v_col;
  const int64_t cols = std::max((H + p.G) * p.DK, vcol + p.GV * p.DV);
  TORCH_CHECK(x.size(1) >= cols, "x has too few columns");
  int64_t rd = 0;
  if (cos_sin.has_value()) {
    TORCH_CHECK(cos_sin->dim() == 2 && cos_sin->size(1) % 2 == 0 && cos_sin->size(1) <= p.DK, "cos_sin must be [max_pos, dims <= DK]");
    rd = cos_sin->size(1);
  }
  TORCH_CHECK(!(q_norm.has_value() || k_norm.has_value() || norm_v) || (dim >= 1 && dim <= p.DK && vdim >= 1 && vdim <= p.DV),
              "norms are over the real dimensions");
  check_rc(pa_paged_kv(f, x.data_ptr(), opt_f32(bias, cols, "bias"), q.data_ptr(), kp.data_ptr(), vp.data_ptr(),
                       pk.data_ptr(), pv.data_ptr(), ints(positions, T, "positions"), ints(slots, T, "slots"),
                       ints(q_start, S, "q_start"), ints(q_len, S, "q_len"), ints(ctx_len, S, "ctx_len"),
                       ints(block_table, 0, "block_table"), opt_f32(cos_sin, 0, "cos_sin"), x.stride(0), H, p.G, p.GV, p.DK,
                       p.DV, rd, pool, p.npb, block_table.size(1), S, T, vcol, opt_f32(q_norm, p.DK, "q_norm"),
                       opt_f32(k_norm, p.DK, "k_norm"), norm_v ? 1 : 0, dim, vdim, (float)eps, cur_stream()),
           "paged_kv");
}

// [T, H, D] whose rows may be part of longer ones
void check_heads(const at::Tensor& t, at::ScalarType dt, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.dim() == 3 && t.stride(2) == 1 && t.stride(1) == t.size(2) && ((uintptr_t)t.data_ptr() & 7) == 0,
              name, " must be a GPU tensor [T, H, D] of whole heads");
  check_dtype(t, dt, name);
}

void window_attention(at::Tensor out, at::Tensor part_o, at::Tensor part_ml, at::Tensor q, at::Tensor kp, at::Tensor vp,
                      at::Tensor pk, at::Tensor pv, at::Tensor items, at::Tensor n_items, at::Tensor q_start,
                      at::Tensor q_len, at::Tensor ctx_len, at::Tensor block_table, int64_t dec_tokens,
                      int64_t tile_tokens, int64_t window, int64_t pool, int64_t keep, int64_t chunk, double scale, Opt slopes,
                      double cap, Opt sink, Opt gate, double gain, int64_t max_slots, bool simple) {
  const int f = is_f32(q, "q"), of = is_f32(out, "out");
  check_gpu(q, "q");
  check_heads(out, out.scalar_type(), "out");
  TORCH_CHECK(of || !f, "out must be float32 or q's type");
  const Pools p = check_pools(kp, vp, pk, pv, q.scalar_type(), pool);
  TORCH_CHECK(q.dim() == 3 && out.size(0) == q.size(0) && out.size(1) == q.size(1) &&
                  q.size(2) == p.DK && out.size(2) == p.DV && q.size(1) % p.G == 0, "q [T, H, DK], out [T, H, DV]");
  TORCH_CHECK(items.dim() == 2 && items.size(1) == 4, "items must be [n, 4]");
  const int64_t H = q.size(1), S = seqs_of(block_table), mi = items.size(0), NB = (dec_tokens * (H / p.G) + 15) / 16;
  TORCH_CHECK(dec_tokens >= 1 && tile_tokens >= 1 && max_slots >= mi, "window_attention sizes");
  TORCH_CHECK(f || simple || (part_o.numel() >= p.G * max_slots * NB * 16 * p.DV && part_ml.numel() >= p.G * max_slots * NB * 32),
              "partition workspace too small");
  TORCH_CHECK(8 * NB * 16 >= std::min<int64_t>(128, tile_tokens * (H / p.G)), "eight slots must hold a tile's columns");
  int64_t ldg = 0;
  if (gate.has_value()) {
    check_rows(*gate, q.scalar_type(), "gate");
    TORCH_CHECK(gate->size(0) == q.size(0) && gate->size(1) >= H * p.DV && ((uintptr_t)gate->data_ptr() & 7) == 0, "gate must be [T, H * DV]");
    ldg = gate->stride(0);
  }
  check_rc(pa_window_attention(f, out.data_ptr(), of && !f ? 1 : 0, out.stride(0), (float*)opt_f32(part_o, 0, "part_o"),
                               (float*)opt_f32(part_ml, 0, "part_ml"), q.data_ptr(), kp.data_ptr(), vp.data_ptr(), pk.data_ptr(),
                               pv.data_ptr(), ints(items, 0, "items"), ints(n_items, 1, "n_items"), mi, ints(q_start, S, "q_start"),
                               ints(q_len, S, "q_len"), ints(ctx_len, S, "ctx_len"), ints(block_table, 0, "block_table"),
                               block_table.size(1), q.size(0), H, p.G, p.GV, p.DK, p.DV, dec_tokens, tile_tokens, window, pool,
                               p.npb, keep, chunk, max_slots, (float)scale, opt_f32(slopes, H, "slopes"), (float)cap,
                               opt_f32(sink, H, "sink"), gate.has_value() ? gate->data_ptr() : nullptr, ldg, (float)gain,
                               simple ? 1 : 0, cur_stream()),
           "window_attention");
}

void head_difference(at::Tensor a, at::Tensor out, at::Tensor gate, int64_t groups, double lam, double gain, int64_t vdim, double eps) {
  const int f = is_f32(out, "out");
  check_gpu(a, "a");
  check_dtype(a, at::kFloat, "a");
  check_heads(out, out.scalar_type(), "out");
  check_rows(gate, out.scalar_type(), "gate");
  const int64_t T = out.size(0), H = out.size(1), D = out.size(2);
  TORCH_CHECK(a.dim() == 3 && a.size(0) == T && a.size(1) == 2 * H && a.size(2) == D && gate.size(0) == T && gate.size(1) >= H * D,
              "head_difference: a [T, 2 H, D], out [T, H, D], gate [T, H * D]");
  check_rc(pa_head_difference(f, a.data_ptr<float>(), out.data_ptr(), out.stride(0), gate.data_ptr(), gate.stride(0), T, H, groups, D,
                              (float)lam, (float)gain, vdim, (float)eps, cur_stream()),
           "head_difference");
}

void state_scan(at::Tensor proj, at::Tensor u, at::Tensor y, at::Tensor state, at::Tensor ring, at::Tensor work,
                at::Tensor total, at::Tensor conv_w, at::Tensor conv_b, at::Tensor dt_bias, at::Tensor a, at::Tensor d,
                at::Tensor q_start, at::Tensor q_len, at::Tensor ctx_len, at::Tensor state_slot, at::Tensor scan_first,
                at::Tensor items, at::Tensor n_items, int64_t max_items, int64_t seqs, int64_t G, int64_t scan_min) {
  const int f = is_f32(proj, "proj");
  check_rows(proj, proj.scalar_type(), "proj");
  check_rows(y, proj.scalar_type(), "y");
  check_gpu(state, "state");
  check_dtype(state, at::kFloat, "state");
  check_gpu(ring, "ring");
  check_dtype(ring, proj.scalar_type(), "ring");
  TORCH_CHECK(state.dim() == 4 && ring.dim() == 3 && ring.size(0) == state.size(0), "state [slots, H, V, N], ring [slots, rows, channels]");
  const int64_t T = proj.size(0), H = state.size(1), V = state.size(2), N = state.size(3), Cc = H * V + 2 * G * N;
  TORCH_CHECK(G > 0 && H % G == 0 && ring.size(2) == Cc && proj.size(1) >= H * V + Cc + H && proj.stride(0) % 8 == 0,
              "state_scan: projection rows are [z | x | B | C | dt]");
  TORCH_CHECK(y.size(0) == T && y.size(1) >= H * V && y.stride(0) % 8 == 0, "y must be [T, >= H * V]");
  TORCH_CHECK(conv_w.dim() == 2 && conv_w.size(1) == Cc, "conv_w must be [taps, channels]");
  TORCH_CHECK(seqs <= q_start.numel() && items.numel() >= 4 * max_items, "state_scan: sequences and items");
  if (max_items > 0) {
    check_gpu(u, "u");
    check_dtype(u, proj.scalar_type(), "u");
    TORCH_CHECK(u.numel() >= T * Cc, "u must be [T, channels]");
    TORCH_CHECK(f || (work.numel() >= max_items * H * V * N && total.numel() >= max_items * H), "state_scan: workspace too small");
  }
  check_rc(pa_state_scan(f, proj.data_ptr(), proj.stride(0), u.data_ptr(), y.data_ptr(), y.stride(0),
                         state.data_ptr<float>(), ring.data_ptr(), (float*)opt_f32(work, 0, "work"),
                         (float*)opt_f32(total, 0, "total"), opt_f32(conv_w, 0, "conv_w"), opt_f32(conv_b, Cc, "conv_b"),
                         opt_f32(dt_bias, H, "dt_bias"), opt_f32(a, H, "a"), opt_f32(d, H, "d"),
                         ints(q_start, seqs, "q_start"), ints(q_len, seqs, "q_len"), ints(ctx_len, seqs, "ctx_len"),
                         ints(state_slot, seqs, "state_slot"), ints(scan_first, seqs, "scan_first"),
                         ints(items, 0, "items"), ints(n_items, 1, "n_items"), max_items, seqs, H, G, V, N,
                         conv_w.size(0), ring.size(1), scan_min, cur_stream()),
           "state_scan");
}

void matrix_memory(at::Tensor x, at::Tensor y, at::Tensor div, at::Tensor state, at::Tensor top, at::Tensor work, at::Tensor stat,
                   at::Tensor i_bias, at::Tensor f_bias, at::Tensor q_start, at::Tensor q_len, at::Tensor ctx_len,
                   at::Tensor state_slot, at::Tensor items, at::Tensor n_items, int64_t max_items, int64_t seqs,
                   std::vector<int64_t> cols, int64_t vdim, double cap, double q_scale, int64_t scan_min) {
  const int f = is_f32(x, "x");
  check_rows(x, x.scalar_type(), "x");
  check_rows(y, x.scalar_type(), "y");
  for (auto* t : {&div, &state, &top, &work, &stat}) {
    check_gpu(*t, "a state");
    check_dtype(*t, at::kFloat, "a state");
  }
  TORCH_CHECK(state.dim() == 4 && top.dim() == 3 && top.size(0) == state.size(0) && top.size(1) == state.size(1) &&
                  top.size(2) == state.size(2), "state [slots, H, V, N], top [slots, H, V]");
  TORCH_CHECK(cols.size() == 5, "cols: q, k, v, gates, width of a value head");
  const int64_t T = x.size(0), H = state.size(1), V = state.size(2), N = state.size(3), vin = cols[4], C = x.size(1);
  TORCH_CHECK(cols[0] >= 0 && cols[0] + H * N <= C && cols[1] >= 0 && cols[1] + H * N <= C && cols[2] >= 0 &&
                  cols[2] + H * vin <= C && cols[3] >= 0 && cols[3] + 2 * H <= C, "x has too few columns");
  TORCH_CHECK(y.size(0) == T && y.size(1) >= H * vin && div.numel() >= T * H, "y must be [T, >= H * vin], div [T, H]");
  TORCH_CHECK(f || (((uintptr_t)x.data_ptr() & 15) == 0 && ((uintptr_t)y.data_ptr() & 7) == 0), "16-byte aligned rows");
  TORCH_CHECK(seqs <= q_start.numel() && items.numel() >= 4 * max_items, "matrix_memory: sequences and items");
  TORCH_CHECK(f || (work.numel() >= max_items * H * V * N && stat.numel() >= max_items * H * 4), "matrix_memory: workspace too small");
  check_rc(pa_matrix_memory(f, x.data_ptr(), x.stride(0), y.data_ptr(), y.stride(0), div.data_ptr<float>(), state.data_ptr<float>(),
                            top.data_ptr<float>(), work.data_ptr<float>(), stat.data_ptr<float>(), opt_f32(i_bias, H, "i_bias"),
                            opt_f32(f_bias, H, "f_bias"), ints(q_start, seqs, "q_start"), ints(q_len, seqs, "q_len"),
                            ints(ctx_len, seqs, "ctx_len"), ints(state_slot, seqs, "state_slot"), ints(items, 0, "items"),
                            ints(n_items, 1, "n_items"), max_items, seqs, H, V, N, cols[0], cols[1], cols[2], cols[3], vin, vdim,
                            (float)cap, (float)q_scale, scan_min, cur_stream()),
           "matrix_memory");
}

}  // namespace

PYBIND11_MODULE(_hybrid, m) {
  m.doc() = "pilottai_amd CDNA4 (gfx950) kernels: paged attention, recurrent layers, score-routed experts";
  m.def("hyper_norm", &hyper_norm);
  m.def("softcap", &softcap);
  m.def("paged_kv", &paged_kv);
  m.def("window_pad", [](int k, int v) {
    int a = 0, b = 0;
    pa_window_pad(k, v, &a, &b);
    return std::make_pair(a, b);
  });
  m.def("window_attention", &window_attention);
  m.def("head_difference", &head_difference);
  m.def("matrix_memory", &matrix_memory);
  m.def("state_scan", &state_scan);
  m.def("gated_norm", &gated_norm);
  m.def("score_route", &score_route);
  m.def("head_gemm", &head_gemm);
  m.def("table_gemm", &table_gemm);
  m.def("expert_gemm", &expert_gemm);
  m.def("empty_uncached", &empty_uncached);
  m.def("decode_gemm", &decode_gemm);
  m.def("prefill_gemm", &prefill_gemm);
}
