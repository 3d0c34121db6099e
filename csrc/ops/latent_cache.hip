// Latent attention's down-projection output -> normed query latent + paged latent cache.
//
// Input row t: [query latent (NQ) | key-value latent (R) | shared key part (r)] of one projection.
//   cq[t]        = norm(query latent) * w_q                      (columns NQ .. ldq zero)
//   page[slot]   = norm(kv latent) * w_c, dims 0 .. R
//                  rotate-half of the key part by the token's position, dims Rp .. Rp + r
// The page layout is fragment-major like the K pages of rope_cache.hip: [D/8][16 keys][8 dims],
// D = Rp + rp, with R and r padded to whole MFMA chunks; the padding is written as zeros, so a
// page needs no initialisation. One copy serves as keys and as values (latent_attention.hip).
#include "common.h"

namespace pa {

template <typename T>
__global__ __launch_bounds__(256) void latent_cache_kernel(
    const T* __restrict__ x, int ldx, int NQ, int R, int r, int rd, const float* __restrict__ w_q,
    const float* __restrict__ w_c, T* __restrict__ cq, int ldq, T* __restrict__ pages, int Rp, int D,
    const int* __restrict__ positions, const int* __restrict__ slots, const float* __restrict__ cos_sin,
    float eps) {
  __shared__ float red[4];
  const int t = blockIdx.x;
  const T* row = x + (size_t)t * ldx;
  float sq = 0.f, sc = 0.f;
  for (int i = threadIdx.x; i < NQ; i += 256) {
    const float v = (float)row[i];
    sq += v * v;
  }
  for (int i = threadIdx.x; i < R; i += 256) {
    const float v = (float)row[NQ + i];
    sc += v * v;
  }
  const float iq = 1.f / sqrtf(block_sum<4>(sq, red) / (float)NQ + eps);
  const float ic = 1.f / sqrtf(block_sum<4>(sc, red) / (float)R + eps);
  T* q = cq + (size_t)t * ldq;
  for (int i = threadIdx.x; i < ldq; i += 256) q[i] = i < NQ ? (T)((float)row[i] * iq * w_q[i]) : (T)0.f;
  const int slot = slots[t];
  if (slot < 0) return;
  T* page = pages + ((size_t)(slot >> 4) * D) * 16 + (slot & 15) * 8;
  const T* kr = row + NQ + R;
  const float* cs = cos_sin + (size_t)positions[t] * rd;
  const int half = rd >> 1;
  for (int i = threadIdx.x; i < D; i += 256) {
    float v = 0.f;
    if (i < R) {
      v = (float)row[NQ + i] * ic * w_c[i];
    } else if (i >= Rp && i - Rp < r) {
      const int j = i - Rp;
      v = (float)kr[j];
      if (j < half) v = v * cs[j] - (float)kr[j + half] * cs[half + j];
      else if (j < rd) v = v * cs[j - half] + (float)kr[j - half] * cs[j];
    }
    page[(size_t)(i >> 3) * 128 + (i & 7)] = (T)v;
  }
}

}  // namespace pa

extern "C" int pa_latent_cache(int fp32, const void* x, int ldx, int NQ, int R, int r, int rd, const float* w_q,
                               const float* w_c, void* cq, int ldq, void* pages, int Rp, int D, const int* positions,
                               const int* slots, const float* cos_sin, float eps, int T, hipStream_t st) {
  if (T <= 0) return 0;
#define PA_LC(TT)                                                                                                \
  hipLaunchKernelGGL((pa::latent_cache_kernel<TT>), dim3(T), dim3(256), 0, st, (const TT*)x, ldx, NQ, R, r, rd,  \
                     w_q, w_c, (TT*)cq, ldq, (TT*)pages, Rp, D, positions, slots, cos_sin, eps)
  if (fp32) PA_LC(float); else PA_LC(pa::bf16);
#undef PA_LC
  return (int)hipGetLastError();
}
