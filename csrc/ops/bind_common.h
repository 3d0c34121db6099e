// Shared by the extension modules' bindings: argument checks, the packed-weight projections that
// every model uses, and uncached hand-off buffers.
#pragma once
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>
#include <hip/hip_runtime_api.h>

#include <map>
#include <mutex>
#include <utility>

extern "C" {
int pa_decode_gemm(void* y, const void* x, const void* wp, const void* resid, int M, int N, int K,
                   int ldx, int ldy, int ldr, int epi, int norm, float eps, int nt, int waves, int splits,
                   float* ws, long long ws_floats, int* counters, int n_counters, hipStream_t st);
int pa_prefill_gemm(void* y, const void* x, const void* wp, const void* resid, float* ws, long long ws_floats,
                    int* counters, int n_counters, int M, int N, int K, int ldx, int ldy, int ldr, int epi,
                    const float* ss_in, float* ss_out, float* ss_zero, float eps, int full, int splits, int bn,
                    void* q_out, void* k_cache, void* v_cache, const int* positions, const int* slots,
                    const float* cos_sin, int H, int KV, int kernel_variant, hipStream_t st);
}

namespace {

hipStream_t cur_stream() { return c10::hip::getCurrentHIPStream().stream(); }

void check_gpu(const at::Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda(), name, " must be a GPU tensor");
  TORCH_CHECK(t.is_contiguous(), name, " must be contiguous");
}

void check_dtype(const at::Tensor& t, at::ScalarType dt, const char* name) {
  TORCH_CHECK(t.scalar_type() == dt, name, " has dtype ", t.scalar_type(), ", expected ", dt);
}

void check_rc(int rc, const char* what) {
  TORCH_CHECK(rc == 0, what, " launch failed with code ", rc, " (",
              rc > 0 ? hipGetErrorString((hipError_t)rc) : "bad arguments", ")");
}

const float* opt_rows(const c10::optional<at::Tensor>& t, int M, const char* name) {
  if (!t.has_value()) return nullptr;
  check_gpu(*t, name);
  check_dtype(*t, at::kFloat, name);
  TORCH_CHECK(t->numel() >= M, name, " must hold >= M floats");
  return t->data_ptr<float>();
}

// y = epi(rownorm(x) . W^T) on fragment-major packed weights wp [N/16, K/32, 64, 8]
// (csrc/ops/gemm_decode.hip). epi 0 plain, 1 silu(gate)*up (y has N/2 columns),
// 2 y = resid + acc. Returns false if the shape is not handled.
bool decode_gemm(at::Tensor y, at::Tensor x, at::Tensor wp, c10::optional<at::Tensor> resid, int64_t epi,
                 bool norm, double eps, int64_t nt, int64_t waves, int64_t splits, c10::optional<at::Tensor> ws,
                 c10::optional<at::Tensor> counters) {
  check_gpu(wp, "wp");
  TORCH_CHECK(x.is_cuda() && x.dim() == 2 && x.stride(1) == 1, "x must be a 2-D GPU tensor, unit inner stride");
  TORCH_CHECK(y.is_cuda() && y.dim() == 2 && y.stride(1) == 1, "y must be a 2-D GPU tensor, unit inner stride");
  check_dtype(x, at::kBFloat16, "x"); check_dtype(wp, at::kBFloat16, "wp"); check_dtype(y, at::kBFloat16, "y");
  TORCH_CHECK(wp.dim() == 4 && wp.size(2) == 64 && wp.size(3) == 8, "wp must be packed [N/16, K/32, 64, 8]");
  const int M = x.size(0), K = x.size(1), N = wp.size(0) * 16;
  TORCH_CHECK(wp.size(1) * 32 == K, "packed weight K ", wp.size(1) * 32, " != x K ", K);
  TORCH_CHECK(x.stride(0) % 8 == 0 && K % 8 == 0, "x rows must be 16-byte aligned");
  const int NO = epi == 1 ? N / 2 : N;
  TORCH_CHECK(y.size(0) == M && y.size(1) == NO, "y shape [", y.size(0), ", ", y.size(1), "] != [", M, ", ", NO, "]");
  const void* rp = nullptr;
  int ldr = 0;
  if (epi == 2) {
    TORCH_CHECK(resid.has_value(), "epi=2 needs resid");
    const auto& r = *resid;
    TORCH_CHECK(r.is_cuda() && r.dim() == 2 && r.stride(1) == 1 && r.size(0) == M && r.size(1) == N,
                "resid must be [M, N] with unit inner stride");
    check_dtype(r, at::kBFloat16, "resid");
    rp = r.data_ptr();
    ldr = r.stride(0);
  }
  float* wsp = nullptr;
  long long wsn = 0;
  int* cp = nullptr;
  int cn = 0;
  if (ws.has_value() && counters.has_value()) {
    check_gpu(*ws, "ws"); check_gpu(*counters, "counters");
    check_dtype(*ws, at::kFloat, "ws"); check_dtype(*counters, at::kInt, "counters");
    wsp = ws->data_ptr<float>(); wsn = ws->numel(); cp = counters->data_ptr<int>(); cn = counters->numel();
  }
  const int rc = pa_decode_gemm(y.data_ptr(), x.data_ptr(), wp.data_ptr(), rp, M, N, K, x.stride(0), y.stride(0),
                                ldr, (int)epi, norm ? 1 : 0, (float)eps, (int)nt, (int)waves, (int)splits, wsp, wsn,
                                cp, cn, cur_stream());
  TORCH_CHECK(rc >= 0, "decode_gemm launch failed");
  return rc == 0;
}

// Large-M projections (csrc/ops/gemm_prefill.hip): 256x256 MFMA tiles on the packed
// weights with the same epilogues as mid_gemm (0 plain, 1 SwiGLU, 2 residual, 3 rope-perm).
bool prefill_gemm(at::Tensor y, at::Tensor x, at::Tensor wp, c10::optional<at::Tensor> resid, at::Tensor ws,
                  at::Tensor counters, int64_t epi, c10::optional<at::Tensor> ss_in, c10::optional<at::Tensor> ss_out,
                  c10::optional<at::Tensor> ss_zero, double eps, int64_t full, int64_t splits, int64_t bn,
                  int64_t variant) {
  check_gpu(wp, "wp"); check_gpu(ws, "ws"); check_gpu(counters, "counters");
  TORCH_CHECK(x.is_cuda() && x.dim() == 2 && x.stride(1) == 1, "x must be a 2-D GPU tensor, unit inner stride");
  TORCH_CHECK(y.is_cuda() && y.dim() == 2 && y.stride(1) == 1, "y must be a 2-D GPU tensor, unit inner stride");
  check_dtype(x, at::kBFloat16, "x"); check_dtype(wp, at::kBFloat16, "wp"); check_dtype(y, at::kBFloat16, "y");
  check_dtype(ws, at::kFloat, "ws"); check_dtype(counters, at::kInt, "counters");
  TORCH_CHECK(epi >= 0 && epi <= 3, "prefill_gemm epi must be 0..3 (RoPE + KV write: prefill_qkv_rope)");
  TORCH_CHECK(wp.dim() == 4 && wp.size(2) == 64 && wp.size(3) == 8, "wp must be packed [N/16, K/32, 64, 8]");
  const int M = x.size(0), K = x.size(1), N = wp.size(0) * 16;
  TORCH_CHECK(wp.size(1) * 32 == K, "packed weight K mismatch");
  TORCH_CHECK(x.stride(0) % 8 == 0 && y.stride(0) % 4 == 0, "x rows must be 16-byte, y rows 8-byte aligned");
  // the non-pair epilogues (plain, residual) of the ping-pong kernels store -- and read the
  // residual -- 16 B per lane (packed_epi.h store_pair_wide): y and resid rows 16-byte aligned
  const bool wide = epi == 0 || epi == 2;
  auto rows16 = [](const at::Tensor& t) { return t.stride(0) % 8 == 0 && ((uintptr_t)t.data_ptr() & 15) == 0; };
  TORCH_CHECK(!wide || rows16(y), "y rows must be 16-byte aligned for the plain / residual epilogue");
  TORCH_CHECK(((uintptr_t)y.data_ptr() & 7) == 0, "y must be 8-byte aligned");
  const int NO = epi == 1 ? N / 2 : N;
  TORCH_CHECK(y.size(0) == M && y.size(1) == NO, "y shape mismatch");
  const void* rp = nullptr;
  int ldr = 0;
  if (epi == 2) {
    TORCH_CHECK(resid.has_value(), "epi=2 needs resid");
    const auto& r = *resid;
    TORCH_CHECK(r.is_cuda() && r.dim() == 2 && r.stride(1) == 1 && r.size(0) == M && r.size(1) == N && rows16(r),
                "resid must be [M, N] with unit inner stride and 16-byte aligned rows");
    check_dtype(r, at::kBFloat16, "resid");
    rp = r.data_ptr();
    ldr = r.stride(0);
  }
  const int rc = pa_prefill_gemm(y.data_ptr(), x.data_ptr(), wp.data_ptr(), rp, ws.data_ptr<float>(), ws.numel(),
                                 counters.data_ptr<int>(), counters.numel(), M, N, K, x.stride(0), y.stride(0), ldr,
                                 (int)epi, opt_rows(ss_in, M, "ss_in"), const_cast<float*>(opt_rows(ss_out, M, "ss_out")),
                                 const_cast<float*>(opt_rows(ss_zero, M, "ss_zero")), (float)eps, (int)full,
                                 (int)splits, (int)bn, nullptr, nullptr, nullptr, nullptr, nullptr, nullptr, 0, 0,
                                 (int)variant, cur_stream());
  TORCH_CHECK(rc >= 0, "prefill_gemm launch failed");
  return rc == 0;
}

// ---- uncached device memory (in-launch hand-off workspaces) ----
// Split-K slabs and attention partials are written by one workgroup and read by another
// inside the same launch. In uncached memory (MTYPE UC: no L1/L2 copy of any line) a reader
// can never see a stale copy held by its own CU or XCD, whatever the placement, so the
// hand-off needs no L2 write-back on the producer side. Such memory is never given back to the
// driver: tensors allocated where an uncached buffer was freed have held wrong values, so a
// released buffer waits here for the next request of its size.
struct UncachedPool {
  std::mutex mu;
  std::multimap<std::pair<int64_t, int64_t>, void*> free;  // (device, bytes) -> buffer
};

inline UncachedPool& uncached_pool() {
  static UncachedPool* p = new UncachedPool;  // outlives every tensor
  return *p;
}

at::Tensor empty_uncached(int64_t numel, at::ScalarType dtype, int64_t device) {
  TORCH_CHECK(numel > 0, "empty_uncached: numel must be positive");
  const int64_t want = numel * (int64_t)c10::elementSize(dtype), grain = (int64_t)1 << 20;
  const int64_t bytes = (want + grain - 1) / grain * grain;
  int prev = 0;
  TORCH_CHECK(hipGetDevice(&prev) == hipSuccess, "hipGetDevice failed");
  TORCH_CHECK(hipSetDevice((int)device) == hipSuccess, "hipSetDevice failed");
  void* p = nullptr;
  {
    UncachedPool& pool = uncached_pool();
    std::lock_guard<std::mutex> g(pool.mu);
    auto it = pool.free.find({device, bytes});
    if (it != pool.free.end()) {
      p = it->second;
      pool.free.erase(it);
    }
  }
  hipError_t e = hipSuccess;
  if (!p) e = hipExtMallocWithFlags(&p, (size_t)bytes, hipDeviceMallocUncached);
  else e = hipDeviceSynchronize();  // its last user's kernels
  if (e == hipSuccess) (void)hipMemset(p, 0, (size_t)bytes);
  (void)hipSetDevice(prev);
  TORCH_CHECK(e == hipSuccess && p != nullptr, "empty_uncached: hipExtMallocWithFlags(", bytes,
              " bytes, uncached) failed");
  TORCH_CHECK(hipDeviceSynchronize() == hipSuccess, "empty_uncached: memset failed");
  auto opts = at::TensorOptions().dtype(dtype).device(at::Device(at::kCUDA, (int)device));
  return torch::from_blob(p, {numel}, [device, bytes](void* q) {
    UncachedPool& pool = uncached_pool();
    std::lock_guard<std::mutex> g(pool.mu);
    pool.free.emplace(std::make_pair(device, bytes), q);
  }, opts);
}

}  // namespace
