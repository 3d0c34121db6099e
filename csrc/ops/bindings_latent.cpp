// Python bindings of the latent-attention / expert-table kernels (module _latent): the kernels a
// model with an fp32 residual stream, latent attention and table-routed experts runs, beside the
// packed-weight projections it shares with the other models. Built as its own module so that such
// a model needs no other kernel. Every entry point checks shapes on the host and launches on the
// caller's stream.
#include "bind_latent.h"

extern "C" {
int pa_table_route(const int* tables, const int* desc, int layers, const int* ids, const int* slots, int T, int tm,
                   int* order, int* tiles, int* n_tiles, hipStream_t st);
}


namespace {

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
  m.def("table_gemm", &table_gemm);
  m.def("expert_gemm", &expert_gemm);
  m.def("empty_uncached", &empty_uncached);
  m.def("decode_gemm", &decode_gemm);
  m.def("prefill_gemm", &prefill_gemm);
}
