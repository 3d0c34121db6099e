// The step between two sublayers of a decoder that keeps its residual stream in fp32 and may
// norm a sublayer's output before adding it:
//
//   r <- r + norm(sum_k y_k * y_scale) * w_post     (or r + sum_k y_k * y_scale without w_post)
//   r <- r + E[id]  or  r <- E[id]                  (embedding rows, added or set)
//   out = norm(r) * w_next                          (the next sublayer's input)
//
// in one launch: one workgroup per row, the row in LDS between the passes, so y, r and the
// embedding row are read once and r and out written once. y is [T, K, ldy] (K partial outputs
// per token, e.g. of its experts). All arithmetic is fp32; y, E and out are T (bf16 or fp32).
// out's columns D .. ldo are set to zero (projections read K padded to whole MFMA chunks).
// `rows` (optional): out row i is row rows[i]'s; r itself is then left as it was (a row may be named
// more than once, by padding).
#include "common.h"

namespace pa {

template <typename T, int VEC>
__global__ __launch_bounds__(256) void residual_norm_kernel(
    float* __restrict__ resid, const T* __restrict__ y, int K, int ldy, float y_scale,
    const float* __restrict__ w_post, const T* __restrict__ emb, const int* __restrict__ ids, int vocab,
    int emb_add, const float* __restrict__ w_next, T* __restrict__ out, int ldo, const int* __restrict__ rows,
    int D, float eps) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[4];
  const int t = rows ? rows[blockIdx.x] : blockIdx.x;
  float* rr = resid + (size_t)t * D;
  float inv = 1.f;
  if (y) {
    const T* yr = y + (size_t)t * K * ldy;
    float ss = 0.f;
    for (int i = threadIdx.x * VEC; i < D; i += 256 * VEC) {
      float v[VEC];
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] = 0.f;
#pragma unroll 4
      for (int k = 0; k < K; ++k) {
        T a[VEC];
        __builtin_memcpy(a, __builtin_assume_aligned(yr + (size_t)k * ldy + i, sizeof(T) * VEC), sizeof(T) * VEC);
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] += (float)a[j];
      }
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        v[j] *= y_scale;
        row[i + j] = v[j];
        ss += v[j] * v[j];
      }
    }
    if (w_post) inv = 1.f / sqrtf(block_sum<4>(ss, red) / (float)D + eps);
  }
  const T* er = nullptr;
  if (emb) er = emb + (size_t)min(max(ids[t], 0), vocab - 1) * D;
  float ss = 0.f;
  for (int i = threadIdx.x * VEC; i < D; i += 256 * VEC) {
    float v[VEC];
    if (er && !emb_add) {
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] = 0.f;
    } else {
      __builtin_memcpy(v, __builtin_assume_aligned(rr + i, 4 * VEC), 4 * VEC);
    }
    if (y) {
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] += w_post ? row[i + j] * inv * w_post[i + j] : row[i + j];
    }
    if (er) {
      T a[VEC];
      __builtin_memcpy(a, __builtin_assume_aligned(er + i, sizeof(T) * VEC), sizeof(T) * VEC);
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] += (float)a[j];
    }
    if ((y || er) && !rows) __builtin_memcpy(__builtin_assume_aligned(rr + i, 4 * VEC), v, 4 * VEC);
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      row[i + j] = v[j];
      ss += v[j] * v[j];
    }
  }
  if (!w_next) return;
  const float inv2 = 1.f / sqrtf(block_sum<4>(ss, red) / (float)D + eps);
  T* o = out + (size_t)blockIdx.x * ldo;
  for (int i = threadIdx.x * VEC; i < D; i += 256 * VEC) {
    T a[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) a[j] = (T)(row[i + j] * inv2 * w_next[i + j]);
    __builtin_memcpy(__builtin_assume_aligned(o + i, sizeof(T) * VEC), a, sizeof(T) * VEC);
  }
  for (int i = D + threadIdx.x; i < ldo; i += 256) o[i] = (T)0.f;
}

}  // namespace pa

extern "C" int pa_residual_norm(int fp32, float* resid, const void* y, int K, int ldy, float y_scale,
                                const float* w_post, const void* emb, const int* ids, int vocab, int emb_add,
                                const float* w_next, void* out, int ldo, const int* rows, int n, int D, float eps,
                                hipStream_t st) {
  if (n <= 0) return 0;
  if (D <= 0 || D * 4 > 96 * 1024) return -1;  // the row in LDS
  const bool vec = D % 8 == 0 && ldy % 8 == 0 && ldo % 8 == 0;
#define PA_RN(T, V)                                                                                        \
  do {                                                                                                     \
    static bool attr = false;                                                                              \
    if (!attr) {                                                                                           \
      (void)hipFuncSetAttribute((const void*)pa::residual_norm_kernel<T, V>,                               \
                                hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024);                    \
      attr = true;                                                                                         \
    }                                                                                                      \
    hipLaunchKernelGGL((pa::residual_norm_kernel<T, V>), dim3(n), dim3(256), (size_t)D * 4, st, resid,     \
                       (const T*)y, K, ldy, y_scale, w_post, (const T*)emb, ids, vocab, emb_add, w_next,   \
                       (T*)out, ldo, rows, D, eps);                                                        \
  } while (0)
  if (fp32) {
    if (vec) PA_RN(float, 8); else PA_RN(float, 1);
  } else {
    if (vec) PA_RN(pa::bf16, 8); else PA_RN(pa::bf16, 1);
  }
#undef PA_RN
  return (int)hipGetLastError();
}
