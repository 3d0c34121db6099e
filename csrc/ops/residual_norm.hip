// The step between two sublayers of a decoder that keeps its residual stream in fp32 and may
// norm a sublayer's output before adding it:
//
//   r <- r + norm(sum_k y_k * y_scale) * w_post     (or r + sum_k y_k * y_scale without w_post)
//   r <- r + E[id]  or  r <- E[id]                  (embedding rows, added or set)
//   X_n <- r,  r <- a_0 E[id] + sum_{0 < j <= n} a_j X_j     (depth average; instead of the line above)
//   out = norm(r) * w_next                          (the next sublayer's input; without w_next r itself)
//
// in one launch: one workgroup per row, the row in LDS between the passes, so y, r and the
// embedding row are read once and r and out written once. y is [T, K, ldy] (K partial outputs
// per token, e.g. of its experts). All arithmetic is fp32; y, E and out are T (bf16 or fp32).
// A norm divides each of `groups` equal parts of the row by the part's own root mean square.
// Depth average: X_1 .. X_(n-1), the results of the layers before, lie in hist [.., T, D], the embedding is X_0, and X_n
// joins them.
// out's columns D .. ldo are set to zero (projections read K padded to whole MFMA chunks).
// `rows` (optional): out row i is row rows[i]'s; r and hist are then left as they were (a row may be named
// more than once, by padding).
#include "common.h"

namespace pa {
namespace rn {

struct Args {
  float* resid;         // [T, D]
  const void* y;        // [T, K, ldy]
  const float* w_post;
  const void* emb;
  const int* ids;
  const float* mix;     // a_0 .. a_n, or null
  float* hist;          // [n, T, D]: X_1 .. X_(n-1), room for X_n
  const float* w_next;
  void* out;
  const int* rows;
  long long hist_step;  // elements from one X to the next
  int K, ldy, vocab, emb_add, n_hist, ldo, D, post_groups, next_groups;
  float y_scale, eps;
};

// 1 / rms of the group an element is in. Threads walk a row in steps of 256 * VEC elements. WHOLE: a wave's
// 64 * VEC elements of a step are of one group (or there is one group): its sum goes to a slot of its own, and a
// group's slots are added. Otherwise a wave per group walks the row in LDS.
template <int VEC, bool WHOLE>
struct GroupNorm {
  float *slots, *inv;
  int groups, len;
  __device__ __forceinline__ void add(int i, float ss) {  // every thread of the wave, once a step
    if constexpr (WHOLE) {
      ss = wave_sum(ss);
      if ((threadIdx.x & 63) == 0) slots[i / (64 * VEC)] = ss;
    }
  }
  __device__ __forceinline__ void finish(const float* row, int D, float eps) {
    __syncthreads();
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    if constexpr (WHOLE) {
      const int n = (D + 64 * VEC - 1) / (64 * VEC), per = groups == 1 ? n : len / (64 * VEC);
      for (int g = threadIdx.x; g < groups; g += 256) {
        float s = 0.f;
        for (int k = 0; k < per; ++k) s += slots[g * per + k];
        inv[g] = 1.f / sqrtf(s / (float)len + eps);
      }
    } else {
      for (int g = wid; g < groups; g += 4) {
        float s = 0.f;
        for (int i = lane; i < len; i += 64) s += row[g * len + i] * row[g * len + i];
        s = wave_sum(s);
        if (lane == 0) inv[g] = 1.f / sqrtf(s / (float)len + eps);
      }
    }
    __syncthreads();
  }
  __device__ __forceinline__ float at(int i) const { return inv[groups == 1 ? 0 : i / len]; }
};

template <typename T, int VEC, bool WHOLE>
__global__ __launch_bounds__(256) void residual_norm_kernel(const Args A) {
  extern __shared__ __attribute__((aligned(16))) float row[];  // [D], slots, groups' factors
  const int D = A.D, t = A.rows ? A.rows[blockIdx.x] : blockIdx.x;
  float* rr = A.resid + (size_t)t * D;
  float* slots = row + (D + 3) / 4 * 4;
  const T* er = A.emb ? (const T*)A.emb + (size_t)min(max(A.ids[t], 0), A.vocab - 1) * D : nullptr;
  const int steps = (D + 256 * VEC - 1) / (256 * VEC);  // (all threads take all steps: waves add up together)
  GroupNorm<VEC, WHOLE> gn{slots, slots + (D + 64 * VEC - 1) / (64 * VEC), A.post_groups, D / A.post_groups};
  if (A.y) {
    const T* yr = (const T*)A.y + (size_t)t * A.K * A.ldy;
    for (int s = 0; s < steps; ++s) {
      const int i = (s * 256 + (int)threadIdx.x) * VEC;
      float ss = 0.f;
      if (i < D) {
        float v[VEC];
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] = 0.f;
#pragma unroll 4
        for (int k = 0; k < A.K; ++k) {
          T a[VEC];
          __builtin_memcpy(a, __builtin_assume_aligned(yr + (size_t)k * A.ldy + i, sizeof(T) * VEC), sizeof(T) * VEC);
#pragma unroll
          for (int j = 0; j < VEC; ++j) v[j] += (float)a[j];
        }
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
          v[j] *= A.y_scale;
          row[i + j] = v[j];
          ss += v[j] * v[j];
        }
      }
      if (A.w_post && (s * 256 + (int)(threadIdx.x & ~63)) * VEC < D) gn.add(i, ss);
    }
    if (A.w_post) gn.finish(row, D, A.eps);
  }
  const float* hr = A.mix ? A.hist + (size_t)t * D : nullptr;
  for (int s = 0; s < steps; ++s) {
    const int i = (s * 256 + (int)threadIdx.x) * VEC;
    float ss = 0.f;
    if (i < D) {
      float v[VEC];
      if (er && !A.emb_add && !A.mix) {
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] = 0.f;
      } else {
        __builtin_memcpy(v, __builtin_assume_aligned(rr + i, 4 * VEC), 4 * VEC);
      }
      if (A.y) {
        const float inv = A.w_post ? gn.at(i) : 1.f;
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] += A.w_post ? row[i + j] * inv * A.w_post[i + j] : row[i + j];
      }
      if (er) {
        T a[VEC];
        __builtin_memcpy(a, __builtin_assume_aligned(er + i, sizeof(T) * VEC), sizeof(T) * VEC);
        if (A.mix) {
          if (!A.rows)
            __builtin_memcpy(__builtin_assume_aligned(A.hist + (A.n_hist - 1) * A.hist_step + (size_t)t * D + i, 4 * VEC), v, 4 * VEC);
          const float a0 = A.mix[0], an = A.mix[A.n_hist];
#pragma unroll
          for (int j = 0; j < VEC; ++j) v[j] = a0 * (float)a[j] + an * v[j];
#pragma unroll 4
          for (int k = 1; k < A.n_hist; ++k) {
            float x[VEC];
            __builtin_memcpy(x, __builtin_assume_aligned(hr + (k - 1) * A.hist_step + i, 4 * VEC), 4 * VEC);
            const float ak = A.mix[k];
#pragma unroll
            for (int j = 0; j < VEC; ++j) v[j] = fmaf(ak, x[j], v[j]);
          }
        } else {
#pragma unroll
          for (int j = 0; j < VEC; ++j) v[j] += (float)a[j];
        }
      }
      if ((A.y || er) && !A.rows) __builtin_memcpy(__builtin_assume_aligned(rr + i, 4 * VEC), v, 4 * VEC);
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        row[i + j] = v[j];
        ss += v[j] * v[j];
      }
    }
    // (the slots of the first norm have been read: its finish ends in a barrier, and its factors lie apart)
    if (A.w_next && (s * 256 + (int)(threadIdx.x & ~63)) * VEC < D) gn.add(i, ss);
  }
  if (!A.out) return;
  if (A.w_next) {
    gn.groups = A.next_groups;
    gn.len = D / A.next_groups;
    gn.finish(row, D, A.eps);
  }
  T* o = (T*)A.out + (size_t)blockIdx.x * A.ldo;
  for (int i = threadIdx.x * VEC; i < D; i += 256 * VEC) {
    T a[VEC];
    const float inv = A.w_next ? gn.at(i) : 1.f;
#pragma unroll
    for (int j = 0; j < VEC; ++j) a[j] = (T)(A.w_next ? row[i + j] * inv * A.w_next[i + j] : row[i + j]);
    __builtin_memcpy(__builtin_assume_aligned(o + i, sizeof(T) * VEC), a, sizeof(T) * VEC);
  }
  for (int i = D + threadIdx.x; i < A.ldo; i += 256) o[i] = (T)0.f;
}

}  // namespace rn
}  // namespace pa

extern "C" int pa_residual_norm(int fp32, float* resid, const void* y, int K, int ldy, float y_scale,
                                const float* w_post, const void* emb, const int* ids, int vocab, int emb_add,
                                const float* mix, float* hist, long long hist_step, int n_hist, const float* w_next,
                                void* out, int ldo, const int* rows, int n, int D, int post_groups, int next_groups,
                                float eps, hipStream_t st) {
  using namespace pa::rn;
  if (n <= 0) return 0;
  if (D <= 0 || D * 4 > 96 * 1024) return -1;  // the row in LDS
  if (post_groups < 1 || next_groups < 1 || D % post_groups || D % next_groups || (mix && (!emb || !hist || n_hist < 1))) return -1;
  const Args A{resid, y, w_post, emb, ids, mix, hist, w_next, out, rows, hist_step, K, ldy, vocab, emb_add, n_hist, ldo, D,
               post_groups, next_groups, y_scale, eps};
  const int most = post_groups > next_groups ? post_groups : next_groups;
  // vectors that divide the groups, so that each lies in one
  auto fits = [&](int v) {
    return D % v == 0 && ldy % v == 0 && ldo % v == 0 && D / post_groups % v == 0 && D / next_groups % v == 0;
  };
  const int vec = fits(8) ? 8 : fits(4) ? 4 : 1;
  auto whole = [&](int g) { return g == 1 || D / g % (64 * vec) == 0; };
  const size_t lds = ((D + 3) / 4 * 4 + (D + 64 * vec - 1) / (64 * vec) + most) * 4;
  if (lds > 159 * 1024) return -1;
#define PA_RN(T, V, W)                                                                              \
  do {                                                                                              \
    static bool attr = false;                                                                       \
    if (!attr) {                                                                                    \
      (void)hipFuncSetAttribute((const void*)residual_norm_kernel<T, V, W>,                         \
                                hipFuncAttributeMaxDynamicSharedMemorySize, 159 * 1024);            \
      attr = true;                                                                                  \
    }                                                                                               \
    hipLaunchKernelGGL((residual_norm_kernel<T, V, W>), dim3(n), dim3(256), lds, st, A);            \
  } while (0)
#define PA_RN_V(T)                                                           \
  do {                                                                       \
    const bool w = whole(post_groups) && whole(next_groups);                 \
    if (vec == 8) { if (w) PA_RN(T, 8, true); else PA_RN(T, 8, false); }     \
    else if (vec == 4) { if (w) PA_RN(T, 4, true); else PA_RN(T, 4, false); } \
    else { if (w) PA_RN(T, 1, true); else PA_RN(T, 1, false); }              \
  } while (0)
  if (fp32) PA_RN_V(float); else PA_RN_V(pa::bf16);
#undef PA_RN_V
#undef PA_RN
  return (int)hipGetLastError();
}
