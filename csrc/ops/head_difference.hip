// Differential attention's second half: the second map's output taken off the first one's, a norm per head without
// a weight, and the output gate.
//
//   a [T, 2 H, D] fp32, heads (KV head g, map, query head r of its group); D padded, vdim real values
//   d = a[g, 0, r] - lam a[g, 1, r];   out[h = g R + r] = gain d / rms(d) sigmoid(gate[h])
//
// One workgroup per token; a power of two of lanes per head, 8 values each.
#include "common.h"

namespace pa {
namespace hd {

template <typename T>
__global__ __launch_bounds__(256) void head_difference_kernel(const float* __restrict__ a, T* __restrict__ out, int ldo,
                                                              const T* __restrict__ gate, int ldg, int H, int R, int D,
                                                              float lam, float gain, float inv_n, float eps) {
  const int t = blockIdx.x, c = D >> 3, bits = 32 - __clz(c - 1);
  for (int u0 = 0; u0 < H << bits; u0 += 256) {
    const int u = u0 + threadIdx.x, h = u >> bits, d = (u & ((1 << bits) - 1)) * 8;
    const bool in = h < H && d < D;
    float v[8], ss = 0.f;
    if (in) {
      const int g = h / R, r = h - g * R;
      const float* p = a + ((size_t)t * 2 * H + (size_t)2 * g * R + r) * D + d;
      float b[8];
      __builtin_memcpy(v, __builtin_assume_aligned(p, 32), 32);
      __builtin_memcpy(b, __builtin_assume_aligned(p + (size_t)R * D, 32), 32);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        v[j] -= lam * b[j];
        ss = fmaf(v[j], v[j], ss);
      }
    }
    for (int m = (1 << bits) >> 1; m > 0; m >>= 1) ss += __shfl_xor(ss, m, 64);
    if (!in) continue;
    const float f = gain / sqrtf(ss * inv_n + eps);
    T z[8];
    __builtin_memcpy(z, __builtin_assume_aligned(gate + (size_t)t * ldg + (size_t)h * D + d, sizeof(T) * 8), sizeof(T) * 8);
#pragma unroll
    for (int j = 0; j < 8; ++j) z[j] = (T)(v[j] * f / (1.f + __expf(-(float)z[j])));
    __builtin_memcpy(__builtin_assume_aligned(out + (size_t)t * ldo + (size_t)h * D + d, sizeof(T) * 8), z, sizeof(T) * 8);
  }
}

}  // namespace hd
}  // namespace pa

extern "C" int pa_head_difference(int fp32, const float* a, void* out, int ldo, const void* gate, int ldg, int T, int H,
                                  int groups, int D, float lam, float gain, int vdim, float eps, hipStream_t st) {
  if (T <= 0) return 0;
  if (groups <= 0 || H % groups || D % 8 || D > 512 || vdim <= 0 || vdim > D || ldo % 8 || ldg % 8) return -1;
  const float inv_n = 1.f / vdim;
  if (fp32) hipLaunchKernelGGL(pa::hd::head_difference_kernel<float>, dim3(T), dim3(256), 0, st, a, (float*)out, ldo, (const float*)gate, ldg, H, H / groups, D, lam, gain, inv_n, eps);
  else hipLaunchKernelGGL(pa::hd::head_difference_kernel<pa::bf16>, dim3(T), dim3(256), 0, st, a, (pa::bf16*)out, ldo, (const pa::bf16*)gate, ldg, H, H / groups, D, lam, gain, inv_n, eps);
  return (int)hipGetLastError();
}
