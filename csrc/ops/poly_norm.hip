// Polynomial norm, an activation of a whole row z of n columns (in place):
//
//   z <- a z / rms(z) + b z^2 / rms(z^2) + c z^3 / rms(z^3) + e        rms(u) = sqrt(mean(u^2) + eps)
//
// with powers element by element: one pass takes the sums of z^2, z^4 and z^6, another writes. One workgroup a row; a
// row of at most NV vectors a thread stays in registers in between. Sums and powers are fp32, z is T (bf16 or fp32).
// Columns n .. cols are set to zero (the next projection reads them against zero weights).
#include "common.h"

namespace pa {
namespace pn {

template <typename T, int VEC, int NV>
__global__ __launch_bounds__(256) void poly_norm_kernel(T* __restrict__ z, int ld, int n, int cols,
                                                        const float* __restrict__ act, float eps) {
  __shared__ float red[3][4];
  T* r = z + (size_t)blockIdx.x * ld;
  struct V { T v[VEC]; };
  V x[NV ? NV : 1];
  auto load = [&](int i) {
    V a;
    __builtin_memcpy(a.v, __builtin_assume_aligned(r + i, sizeof(a.v)), sizeof(a.v));
    return a;
  };
  float s2 = 0.f, s4 = 0.f, s6 = 0.f;
  auto add = [&](const V& a) {
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      const float v = (float)a.v[j], q = v * v, q2 = q * q;
      s2 += q;
      s4 += q2;
      s6 = fmaf(q2, q, s6);
    }
  };
  if constexpr (NV > 0) {
#pragma unroll
    for (int k = 0; k < NV; ++k) {
      const int i = (k * 256 + (int)threadIdx.x) * VEC;
      if (i < n) x[k] = load(i);
    }
#pragma unroll
    for (int k = 0; k < NV; ++k)
      if ((k * 256 + (int)threadIdx.x) * VEC < n) add(x[k]);
  } else {
    for (int i = threadIdx.x * VEC; i < n; i += 256 * VEC) add(load(i));
  }
  s2 = wave_sum(s2);
  s4 = wave_sum(s4);
  s6 = wave_sum(s6);
  if ((threadIdx.x & 63) == 0) {
    const int w = threadIdx.x >> 6;
    red[0][w] = s2;
    red[1][w] = s4;
    red[2][w] = s6;
  }
  __syncthreads();
  auto factor = [&](int k) {
    return act[k] / sqrtf((red[k][0] + red[k][1] + red[k][2] + red[k][3]) / (float)n + eps);
  };
  const float a = factor(0), b = factor(1), c = factor(2), e = act[3];
  auto store = [&](int i, const V& in) {
    V o;
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      const float v = (float)in.v[j];
      o.v[j] = (T)fmaf(fmaf(fmaf(c, v, b), v, a), v, e);
    }
    __builtin_memcpy(__builtin_assume_aligned(r + i, sizeof(o.v)), o.v, sizeof(o.v));
  };
  if constexpr (NV > 0) {
#pragma unroll
    for (int k = 0; k < NV; ++k) {
      const int i = (k * 256 + (int)threadIdx.x) * VEC;
      if (i < n) store(i, x[k]);
    }
  } else {
    for (int i = threadIdx.x * VEC; i < n; i += 256 * VEC) store(i, load(i));
  }
  for (int i = n + threadIdx.x; i < cols; i += 256) r[i] = (T)0.f;
}

}  // namespace pn
}  // namespace pa

extern "C" int pa_poly_norm(int fp32, void* z, int ld, int rows, int n, int cols, const float* act, float eps, hipStream_t st) {
  using namespace pa::pn;
  if (rows <= 0) return 0;
  if (n < 1 || cols < n || cols > ld) return -1;
  const bool vec = n % 8 == 0 && ld % 8 == 0;
  const int nv = !vec ? 0 : n <= 4096 ? 2 : n <= 8192 ? 4 : n <= 16384 ? 8 : 0;
#define PA_PN(T, V, N) hipLaunchKernelGGL((poly_norm_kernel<T, V, N>), dim3(rows), dim3(256), 0, st, (T*)z, ld, n, cols, act, eps)
#define PA_PN_T(T)                                                     \
  do {                                                                 \
    if (!vec) PA_PN(T, 1, 0);                                          \
    else if (nv == 2) PA_PN(T, 8, 2);                                  \
    else if (nv == 4) PA_PN(T, 8, 4);                                  \
    else if (nv == 8) PA_PN(T, 8, 8);                                  \
    else PA_PN(T, 8, 0);                                               \
  } while (0)
  if (fp32) PA_PN_T(float); else PA_PN_T(pa::bf16);
#undef PA_PN_T
#undef PA_PN
  return (int)hipGetLastError();
}
