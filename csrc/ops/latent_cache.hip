// Latent attention's down-projection output -> normed query latent + paged latent cache.
//
// Input row t: [query latent (NQ) | key-value latent (R) | shared key part (r)] of one projection.
//   cq[t]        = norm(query latent) * w_q                      (columns NQ .. ldq zero; NQ 0: none)
//   page[slot]   = norm(kv latent) * w_c, dims 0 .. R
//                  rotate-half of the key part by the token's position, dims Rp .. Rp + r (r 0: none)
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
  const float iq = 1.f / sqrtf(block_sum<4>(sq, red) / (float)max(NQ, 1) + eps);
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

// The same for sizes in whole 8s (and every rotated dimension paired): a wave per row, 8 columns per
// lane and step, no barrier.
template <typename T>
__global__ __launch_bounds__(256) void latent_cache_wave_kernel(
    const T* __restrict__ x, int ldx, int NQ, int R, int r, const float* __restrict__ w_q,
    const float* __restrict__ w_c, T* __restrict__ cq, int ldq, T* __restrict__ pages, int Rp, int D,
    const int* __restrict__ positions, const int* __restrict__ slots, const float* __restrict__ cos_sin, float eps,
    int rows) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (t >= rows) return;
  const T* row = x + (size_t)t * ldx;
  struct V8 { T v[8]; };
  auto load = [](const T* p) {
    V8 a;
    __builtin_memcpy(a.v, __builtin_assume_aligned(p, 16), sizeof(a.v));
    return a;
  };
  auto store = [](T* p, const float (&v)[8]) {
    T a[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) a[j] = (T)v[j];
    __builtin_memcpy(__builtin_assume_aligned(p, 16), a, sizeof(a));
  };
  const int slot = slots[t];
  const float* cs = cos_sin + (size_t)positions[t] * r;
  float sq = 0.f, sc = 0.f;
  for (int i = lane * 8; i < NQ + R; i += 512) {
    const V8 a = load(row + i);
    float e = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) e += (float)a.v[j] * (float)a.v[j];
    if (i < NQ) sq += e;
    else sc += e;
  }
  const float iq = 1.f / sqrtf(wave_sum(sq) / (float)max(NQ, 1) + eps);
  const float ic = 1.f / sqrtf(wave_sum(sc) / (float)R + eps);
  T* q = cq + (size_t)t * ldq;
  for (int i = lane * 8; i < ldq; i += 512) {
    float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (i < NQ) {
      const V8 a = load(row + i);
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] = (float)a.v[j] * iq * w_q[i + j];
    }
    store(q + i, v);
  }
  if (slot < 0) return;
  T* page = pages + ((size_t)(slot >> 4) * D) * 16 + (slot & 15) * 8;
  const T* kr = row + NQ + R;
  const int half = r >> 1;
  for (int i = lane * 8; i < D; i += 512) {
    float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    const int j0 = i - Rp;
    if (i < R) {
      const V8 a = load(row + NQ + i);
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] = (float)a.v[j] * ic * w_c[i + j];
    } else if (j0 >= 0 && j0 < r) {
      const bool lo = j0 < half;
      const int k = lo ? j0 : j0 - half;
      const V8 a = load(kr + k), b = load(kr + half + k);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float c = cs[k + j], s = cs[half + k + j];
        v[j] = lo ? (float)a.v[j] * c - (float)b.v[j] * s : (float)b.v[j] * c + (float)a.v[j] * s;
      }
    }
    store(page + (size_t)i * 16, v);
  }
}

}  // namespace pa

extern "C" int pa_latent_cache(int fp32, const void* x, int ldx, int NQ, int R, int r, int rd, const float* w_q,
                               const float* w_c, void* cq, int ldq, void* pages, int Rp, int D, const int* positions,
                               const int* slots, const float* cos_sin, float eps, int T, hipStream_t st) {
  if (T <= 0) return 0;
  if (NQ % 8 == 0 && R % 8 == 0 && rd == r && r % 16 == 0 && ldx % 8 == 0 && ldq % 8 == 0) {
#define PA_LW(TT)                                                                                               \
  hipLaunchKernelGGL((pa::latent_cache_wave_kernel<TT>), dim3((T + 3) / 4), dim3(256), 0, st, (const TT*)x, ldx, \
                     NQ, R, r, w_q, w_c, (TT*)cq, ldq, (TT*)pages, Rp, D, positions, slots, cos_sin, eps, T)
    if (fp32) PA_LW(float); else PA_LW(pa::bf16);
#undef PA_LW
    return (int)hipGetLastError();
  }
#define PA_LC(TT)                                                                                                \
  hipLaunchKernelGGL((pa::latent_cache_kernel<TT>), dim3(T), dim3(256), 0, st, (const TT*)x, ldx, NQ, R, r, rd,  \
                     w_q, w_c, (TT*)cq, ldq, (TT*)pages, Rp, D, positions, slots, cos_sin, eps)
  if (fp32) PA_LC(float); else PA_LC(pa::bf16);
#undef PA_LC
  return (int)hipGetLastError();
}
