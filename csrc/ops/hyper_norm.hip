// The step between two sublayers of a decoder whose fp32 residual has several streams x_1 .. x_S
// (hyper-connections; S = 1 with unit weights is the plain residual sum):
//
//   y   <- sum_k w_k y_k + y2 + bias                   (K partial outputs per token, weights optional)
//   x_t <- sum_s mix[s][t] x_s + post[t] y              or, at the start, x_t <- E[id]
//   out <- norm(sum_s pre[s] x_s) * w_next              (the next sublayer's input)
//
// in one launch: one workgroup per row; the streams are read and written once, all from the old ones, and
// the next input waits in LDS for its norm. All arithmetic is fp32; y, E and out are T (bf16 or fp32).
// out's columns D .. ldo are set to zero (projections read K padded to whole MFMA chunks). `rows`
// (optional): out row i is row rows[i]'s, and x is left as it was.
//
// Also here: the soft cap of logits, z <- cap * tanh(z / cap).
#include "common.h"

namespace pa {
namespace hn {

constexpr int MAX_S = 8;

struct Args {
  float* x;             // [T, S, D]
  const void* y;        // [T, K, ldy]
  const float* y_w;     // [T, K] or null
  const void* y2;       // [T, ldy2] or null
  const float* bias;    // [D] or null
  const float *mix, *post, *pre;  // [S, S] from x to, [S], [S]
  const void* emb;
  const int* ids;
  const float* w_next;
  void* out;
  const int* rows;
  int K, ldy, ldy2, vocab, ldo, D;
  float eps;
};

template <typename T, int VEC, int S>
__global__ __launch_bounds__(256) void hyper_norm_kernel(const Args A) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[4];
  const int t = A.rows ? A.rows[blockIdx.x] : blockIdx.x, D = A.D;
  float* xr = A.x + (size_t)t * S * D;
  float mix[S][S], post[S], pre[S];
#pragma unroll
  for (int s = 0; s < S; ++s) {
    pre[s] = A.pre ? A.pre[s] : 0.f;
    post[s] = A.y ? A.post[s] : 0.f;
#pragma unroll
    for (int r = 0; r < S; ++r) mix[s][r] = A.y ? A.mix[s * S + r] : 0.f;
  }
  const T* yr = (const T*)A.y + (size_t)t * A.K * A.ldy;
  const float* yw = A.y_w ? A.y_w + (size_t)t * A.K : nullptr;
  const T* er = A.emb ? (const T*)A.emb + (size_t)min(max(A.ids[t], 0), A.vocab - 1) * D : nullptr;
  float ss = 0.f;
  for (int i = threadIdx.x * VEC; i < D; i += 256 * VEC) {
    float x[S][VEC], u[VEC];
    T a[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) u[j] = 0.f;
    if (er) {
      __builtin_memcpy(a, __builtin_assume_aligned(er + i, sizeof(T) * VEC), sizeof(T) * VEC);
#pragma unroll
      for (int s = 0; s < S; ++s)
#pragma unroll
        for (int j = 0; j < VEC; ++j) x[s][j] = (float)a[j];
    } else {
#pragma unroll
      for (int s = 0; s < S; ++s)
        __builtin_memcpy(x[s], __builtin_assume_aligned(xr + (size_t)s * D + i, 4 * VEC), 4 * VEC);
    }
    if (A.y) {
      float y[VEC];
#pragma unroll
      for (int j = 0; j < VEC; ++j) y[j] = A.bias ? A.bias[i + j] : 0.f;
      if (A.y2) {
        __builtin_memcpy(a, __builtin_assume_aligned((const T*)A.y2 + (size_t)t * A.ldy2 + i, sizeof(T) * VEC), sizeof(T) * VEC);
#pragma unroll
        for (int j = 0; j < VEC; ++j) y[j] += (float)a[j];
      }
#pragma unroll 4
      for (int k = 0; k < A.K; ++k) {
        __builtin_memcpy(a, __builtin_assume_aligned(yr + (size_t)k * A.ldy + i, sizeof(T) * VEC), sizeof(T) * VEC);
        const float w = yw ? yw[k] : 1.f;
#pragma unroll
        for (int j = 0; j < VEC; ++j) y[j] = fmaf(w, (float)a[j], y[j]);
      }
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        float z[S];
#pragma unroll
        for (int r = 0; r < S; ++r) {
          z[r] = post[r] * y[j];
#pragma unroll
          for (int s = 0; s < S; ++s) z[r] = fmaf(mix[s][r], x[s][j], z[r]);
        }
#pragma unroll
        for (int r = 0; r < S; ++r) x[r][j] = z[r];
      }
    }
    if ((A.y || er) && !A.rows) {
#pragma unroll
      for (int s = 0; s < S; ++s)
        __builtin_memcpy(__builtin_assume_aligned(xr + (size_t)s * D + i, 4 * VEC), x[s], 4 * VEC);
    }
#pragma unroll
    for (int s = 0; s < S; ++s)
#pragma unroll
      for (int j = 0; j < VEC; ++j) u[j] = fmaf(pre[s], x[s][j], u[j]);
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      row[i + j] = u[j];
      ss += u[j] * u[j];
    }
  }
  if (!A.w_next) return;
  const float inv = 1.f / sqrtf(block_sum<4>(ss, red) / (float)D + A.eps);
  T* o = (T*)A.out + (size_t)blockIdx.x * A.ldo;
  for (int i = threadIdx.x * VEC; i < D; i += 256 * VEC) {
    T a[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) a[j] = (T)(row[i + j] * inv * A.w_next[i + j]);
    __builtin_memcpy(__builtin_assume_aligned(o + i, sizeof(T) * VEC), a, sizeof(T) * VEC);
  }
  for (int i = D + threadIdx.x; i < A.ldo; i += 256) o[i] = (T)0.f;
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void softcap_kernel(T* __restrict__ x, int ld, int cols, float cap) {
  T* r = x + (size_t)blockIdx.y * ld;
  for (int i = (blockIdx.x * 256 + threadIdx.x) * VEC; i < cols; i += gridDim.x * 256 * VEC) {
    T a[VEC];  // (columns behind cols, up to a whole vector of the row, are padding)
    __builtin_memcpy(a, __builtin_assume_aligned(r + i, sizeof(T) * VEC), sizeof(T) * VEC);
#pragma unroll
    for (int j = 0; j < VEC; ++j)
      if (VEC == 1 || i + j < cols) a[j] = (T)(cap * tanhf((float)a[j] / cap));
    __builtin_memcpy(__builtin_assume_aligned(r + i, sizeof(T) * VEC), a, sizeof(T) * VEC);
  }
}

}  // namespace hn
}  // namespace pa

extern "C" int pa_hyper_norm(int fp32, float* x, int S, const void* y, int K, int ldy, const float* y_w,
                             const void* y2, int ldy2, const float* bias, const float* mix, const float* post, const float* pre, const void* emb,
                             const int* ids, int vocab, const float* w_next, void* out, int ldo, const int* rows, int n,
                             int D, float eps, hipStream_t st) {
  using namespace pa::hn;
  if (n <= 0) return 0;
  if (D <= 0 || D * 4 > 96 * 1024 || S < 1 || S > MAX_S) return -1;
  const Args A{x, y, y_w, y2, bias, mix, post, pre, emb, ids, w_next, out, rows, K, ldy, ldy2, vocab, ldo, D, eps};
  const bool vec = D % 4 == 0 && (!y || ldy % 4 == 0) && (!y2 || ldy2 % 4 == 0) && (!out || ldo % 4 == 0);
#define PA_HN(T, V, N)                                                                                          \
  do {                                                                                                          \
    static bool attr = false;                                                                                   \
    if (!attr) {                                                                                                \
      (void)hipFuncSetAttribute((const void*)hyper_norm_kernel<T, V, N>,                                        \
                                hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024);                         \
      attr = true;                                                                                              \
    }                                                                                                           \
    hipLaunchKernelGGL((hyper_norm_kernel<T, V, N>), dim3(n), dim3(256), (size_t)D * 4, st, A);                 \
  } while (0)
#define PA_HN_S(N)                                                             \
  case N:                                                                      \
    if (fp32) { if (vec) PA_HN(float, 4, N); else PA_HN(float, 1, N); }        \
    else { if (vec) PA_HN(pa::bf16, 4, N); else PA_HN(pa::bf16, 1, N); }       \
    break
  switch (S) {
    PA_HN_S(1); PA_HN_S(2); PA_HN_S(3); PA_HN_S(4); PA_HN_S(5); PA_HN_S(6); PA_HN_S(7); PA_HN_S(8);
  }
#undef PA_HN_S
#undef PA_HN
  return (int)hipGetLastError();
}

extern "C" int pa_softcap(int fp32, void* x, int ld, int rows, int cols, float cap, hipStream_t st) {
  if (rows <= 0 || cols <= 0) return 0;
  const bool vec = ld % 8 == 0;  // (a whole vector then never leaves the row)
  const dim3 grid((cols + 2047) / 2048, rows);
  if (fp32) {
    if (vec) hipLaunchKernelGGL((pa::hn::softcap_kernel<float, 8>), grid, dim3(256), 0, st, (float*)x, ld, cols, cap);
    else hipLaunchKernelGGL((pa::hn::softcap_kernel<float, 1>), grid, dim3(256), 0, st, (float*)x, ld, cols, cap);
  } else {
    if (vec) hipLaunchKernelGGL((pa::hn::softcap_kernel<pa::bf16, 8>), grid, dim3(256), 0, st, (pa::bf16*)x, ld, cols, cap);
    else hipLaunchKernelGGL((pa::hn::softcap_kernel<pa::bf16, 1>), grid, dim3(256), 0, st, (pa::bf16*)x, ld, cols, cap);
  }
  return (int)hipGetLastError();
}
