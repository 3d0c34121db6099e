// The norm behind a recurrence: y, normed in equal parts of the unpadded columns, times w and a gate, in place.
//   after 0   y <- norm(y silu(z)) w
//   after 1   y <- norm(y) w sigmoid(z)
//   after 2   y <- norm(y) w silu(z)
// y's columns are h * Vp + v (v < V) of `cols`; one workgroup per token. With div [T, H] a head is divided by it first.
#include "common.h"

namespace pa {
namespace gn {

enum { BEFORE = 0, SIGMOID_AFTER = 1, SILU_AFTER = 2 };

__device__ __forceinline__ float silu(float x) { return x / (1.f + __expf(-x)); }

template <typename T>
__global__ __launch_bounds__(256) void gated_norm_kernel(T* __restrict__ y, int ldy, int cols, const T* __restrict__ z, int ldz,
                                                         const float* __restrict__ w, const int* __restrict__ slots,
                                                         const float* __restrict__ div, int after, int H, int V, int Vp,
                                                         int parts, float eps) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[4];
  const int t = blockIdx.x, inner = H * V, len = inner / parts;
  if (slots[t] < 0) return;
  T* yr = y + (size_t)t * ldy;
  const T* zr = z + (size_t)t * ldz;
  const int wid = threadIdx.x >> 6, lane = threadIdx.x & 63;
  auto col = [&](int i) { return V == Vp ? i : i / V * Vp + i % V; };
  // what the norm is taken of: the gate ahead of it and the division, by column i's head
  auto inv_div = [&](int i) { return div ? 1.f / div[(size_t)t * H + i / V] : 1.f; };
  auto lead = [&](float v, float g, float f) { return (after ? v : v * silu(g)) * f; };
  auto gate = [&](float g) { return after == SILU_AFTER ? silu(g) : after ? 1.f / (1.f + __expf(-g)) : 1.f; };
  if (V == Vp) {
    for (int i = threadIdx.x * 8; i < inner; i += 2048) {  // (8 columns of one head: Vp is a multiple of 8)
      T a[8], b[8];
      const float f = inv_div(i);
      __builtin_memcpy(a, __builtin_assume_aligned(yr + i, sizeof(T) * 8), sizeof(T) * 8);
      if (!after) __builtin_memcpy(b, __builtin_assume_aligned(zr + i, sizeof(T) * 8), sizeof(T) * 8);
#pragma unroll
      for (int j = 0; j < 8; ++j) row[i + j] = lead((float)a[j], after ? 0.f : (float)b[j], f);
    }
  } else {
    for (int i = threadIdx.x; i < inner; i += 256) row[i] = lead((float)yr[col(i)], (float)zr[col(i)], inv_div(i));
  }
  __syncthreads();
  float* inv = row + inner;  // [parts]
  if (parts >= 4) {
    for (int p = wid; p < parts; p += 4) {
      float ss = 0.f;
      for (int i = lane; i < len; i += 64) ss += row[p * len + i] * row[p * len + i];
      ss = wave_sum(ss);
      if (lane == 0) inv[p] = 1.f / sqrtf(ss / (float)len + eps);
    }
  } else {
    for (int p = 0; p < parts; ++p) {
      float ss = 0.f;
      for (int i = threadIdx.x; i < len; i += 256) ss += row[p * len + i] * row[p * len + i];
      ss = block_sum<4>(ss, red);
      if (threadIdx.x == 0) inv[p] = 1.f / sqrtf(ss / (float)len + eps);
    }
  }
  __syncthreads();
  if (V == Vp && len % 8 == 0) {
    for (int i = threadIdx.x * 8; i < inner; i += 2048) {
      const float f = inv[i / len];
      T a[8], b[8];
      if (after) __builtin_memcpy(b, __builtin_assume_aligned(zr + i, sizeof(T) * 8), sizeof(T) * 8);
#pragma unroll
      for (int j = 0; j < 8; ++j) a[j] = (T)(row[i + j] * f * w[i + j] * gate(after ? (float)b[j] : 0.f));
      __builtin_memcpy(__builtin_assume_aligned(yr + i, sizeof(T) * 8), a, sizeof(T) * 8);
    }
  } else {
    for (int i = threadIdx.x; i < inner; i += 256) yr[col(i)] = (T)(row[i] * inv[i / len] * w[i] * gate(after ? (float)zr[col(i)] : 0.f));
    // padded columns meet zero weights, but must be finite
    if (V != Vp)
      for (int i = threadIdx.x; i < H * (Vp - V); i += 256) yr[i / (Vp - V) * Vp + V + i % (Vp - V)] = (T)0.f;
  }
  for (int i = H * Vp + threadIdx.x; i < cols; i += 256) yr[i] = (T)0.f;
}

// The same where a part is a power of two of 8-column units within a wave (and nothing is padded): no LDS.
template <typename T>
__global__ __launch_bounds__(256) void gated_norm_wave_kernel(T* __restrict__ y, int ldy, int cols, const T* __restrict__ z, int ldz,
                                                              const float* __restrict__ w, const int* __restrict__ slots,
                                                              const float* __restrict__ div, int after, int rows, int H, int V,
                                                              int lanes, float eps) {
  const int units = H * V >> 3, u = blockIdx.x * 256 + threadIdx.x, t = u / units, i = (u - t * units) * 8;
  if (t >= rows) return;  // (whole parts)
  T* yr = y + (size_t)t * ldy;
  const bool live = slots[t] >= 0;
  T a[8], b[8];
  float wv[8], v[8], g[8], ss = 0.f;
  __builtin_memcpy(a, __builtin_assume_aligned(yr + i, sizeof(T) * 8), sizeof(T) * 8);
  __builtin_memcpy(b, __builtin_assume_aligned(z + (size_t)t * ldz + i, sizeof(T) * 8), sizeof(T) * 8);
  __builtin_memcpy(wv, __builtin_assume_aligned(w + i, 16), 32);
  const float f = div ? 1.f / div[(size_t)t * H + i / V] : 1.f;
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    g[j] = 1.f / (1.f + __expf(-(float)b[j]));
    v[j] = (float)a[j] * f;
    if (!after) v[j] *= (float)b[j] * g[j];
    ss = fmaf(v[j], v[j], ss);
  }
  for (int m = lanes >> 1; m > 0; m >>= 1) ss += __shfl_xor(ss, m, 64);
  if (!live) return;
  const float inv = 1.f / sqrtf(ss / (float)(lanes * 8) + eps);
#pragma unroll
  for (int j = 0; j < 8; ++j) a[j] = (T)(v[j] * inv * wv[j] * (after == SILU_AFTER ? (float)b[j] * g[j] : after ? g[j] : 1.f));
  __builtin_memcpy(__builtin_assume_aligned(yr + i, sizeof(T) * 8), a, sizeof(T) * 8);
  for (int k = H * V + i / 8; k < cols; k += units) yr[k] = (T)0.f;
}

}  // namespace gn
}  // namespace pa

extern "C" int pa_gated_norm(int fp32, void* y, int ldy, int cols, const void* z, int ldz, const float* w, const int* slots,
                             const float* div, int after, int T, int H, int V, int Vp, int parts, float eps,
                             hipStream_t st) {
  if (T <= 0) return 0;
  if (H * V % parts || Vp % 8 || ldy % 8 || ldz % 8) return -1;
  const int len = H * V / parts, lanes = len / 8;
  if (V == Vp && len % 8 == 0 && lanes <= 64 && (lanes & (lanes - 1)) == 0) {
    const dim3 grid(((long long)T * (H * V / 8) + 255) / 256);
    if (fp32) hipLaunchKernelGGL(pa::gn::gated_norm_wave_kernel<float>, grid, dim3(256), 0, st, (float*)y, ldy, cols, (const float*)z, ldz, w, slots, div, after, T, H, V, lanes, eps);
    else hipLaunchKernelGGL(pa::gn::gated_norm_wave_kernel<pa::bf16>, grid, dim3(256), 0, st, (pa::bf16*)y, ldy, cols, (const pa::bf16*)z, ldz, w, slots, div, after, T, H, V, lanes, eps);
    return (int)hipGetLastError();
  }
  const int lds = (H * V + parts) * 4;
  if (lds > 160 * 1024 - 64) return -2;
  static bool attr = false;
  if (!attr) {
    (void)hipFuncSetAttribute((const void*)pa::gn::gated_norm_kernel<float>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024 - 64);
    (void)hipFuncSetAttribute((const void*)pa::gn::gated_norm_kernel<pa::bf16>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024 - 64);
    attr = true;
  }
  if (fp32) hipLaunchKernelGGL(pa::gn::gated_norm_kernel<float>, dim3(T), dim3(256), lds, st, (float*)y, ldy, cols, (const float*)z, ldz, w, slots, div, after, H, V, Vp, parts, eps);
  else hipLaunchKernelGGL(pa::gn::gated_norm_kernel<pa::bf16>, dim3(T), dim3(256), lds, st, (pa::bf16*)y, ldy, cols, (const pa::bf16*)z, ldz, w, slots, div, after, H, V, Vp, parts, eps);
  return (int)hipGetLastError();
}
