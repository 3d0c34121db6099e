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

#include <type_traits>

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

// The same for rows of whole 8s whose groups are whole wave steps of 512 elements or a power of two of lanes: W waves a row
// (4 / W rows a workgroup), NV vectors a thread in registers, all of a row's loads ahead of the first sum.
template <typename T, int W, int NV>
__global__ __launch_bounds__(256) void residual_norm_wave_kernel(const Args A, int n) {
  constexpr int R = 4 / W;
  __shared__ float slots[W > 1 ? R : 1][W > 1 ? W * NV : 1];
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, w = wid % W, r = wid / W;
  const int b = blockIdx.x * R + r, D = A.D;
  if (W == 1 && b >= n) return;  // (whole waves; with W > 1 all take the barriers)
  const int t = A.rows ? A.rows[min(b, n - 1)] : min(b, n - 1);
  auto at = [&](int s) { return ((s * W + w) * 64 + lane) * 8; };
  auto in = [&](int s) { return min(at(s), D - 8); };  // (loads without branches; past the end they repeat the last 8)
  // 1 / rms of the group of each of a thread's vectors
  auto factors = [&](const float (&ss)[NV], int groups, float (&inv)[NV]) {
    const int len = D / groups, width = groups == 1 ? 64 : min(64, len >> 3), units = groups == 1 ? W * NV : max(1, len >> 9);
    float part[NV];
#pragma unroll
    for (int s = 0; s < NV; ++s) {
      part[s] = ss[s];
      for (int o = width >> 1; o > 0; o >>= 1) part[s] += __shfl_xor(part[s], o, 64);
    }
    if constexpr (W > 1) {
      __syncthreads();
      if (lane == 0) {
#pragma unroll
        for (int s = 0; s < NV; ++s) slots[r][s * W + w] = part[s];
      }
      __syncthreads();
    }
#pragma unroll
    for (int s = 0; s < NV; ++s) {
      float sum = 0.f;
      if (units == 1) {
        sum = part[s];
      } else if constexpr (W > 1) {
        const int u0 = (s * W + w) / units * units;
        for (int u = u0; u < min(u0 + units, W * NV); ++u) sum += slots[r][u];
      } else {
#pragma unroll
        for (int k = 0; k < NV; ++k) sum += k / units == s / units ? part[k] : 0.f;
      }
      inv[s] = 1.f / sqrtf(sum / (float)len + A.eps);
    }
  };
  auto load = [](const auto* p, float (&v)[8]) {
    using E = std::remove_cv_t<std::remove_pointer_t<decltype(p)>>;
    E a[8];
    __builtin_memcpy(a, __builtin_assume_aligned(p, sizeof(E) * 8), sizeof(a));
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = (float)a[j];
  };
  float* rr = A.resid + (size_t)t * D;
  const T* er = A.emb ? (const T*)A.emb + (size_t)min(max(A.ids[t], 0), A.vocab - 1) * D : nullptr;
  const bool set = er && !A.emb_add && !A.mix;
  float y[NV][8], x[NV][8], ss[NV], inv[NV];
#pragma unroll
  for (int s = 0; s < NV; ++s) {
    ss[s] = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) x[s][j] = y[s][j] = 0.f;
    if (!set) load(rr + in(s), x[s]);
  }
  if (A.y) {
    const T* yr = (const T*)A.y + (size_t)t * A.K * A.ldy;
#pragma unroll 4
    for (int k = 0; k < A.K; ++k)
#pragma unroll
      for (int s = 0; s < NV; ++s) {
        float v[8];
        load(yr + (size_t)k * A.ldy + in(s), v);
#pragma unroll
        for (int j = 0; j < 8; ++j) y[s][j] += v[j];
      }
#pragma unroll
    for (int s = 0; s < NV; ++s) {
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        y[s][j] *= A.y_scale;
        ss[s] = fmaf(y[s][j], y[s][j], ss[s]);
      }
      if (at(s) >= D) ss[s] = 0.f;
    }
    if (A.w_post) {
      float g[NV][8];  // (on their way during the sum)
#pragma unroll
      for (int s = 0; s < NV; ++s) load(A.w_post + in(s), g[s]);
      factors(ss, A.post_groups, inv);
#pragma unroll
      for (int s = 0; s < NV; ++s)
#pragma unroll
        for (int j = 0; j < 8; ++j) x[s][j] = fmaf(y[s][j] * inv[s], g[s][j], x[s][j]);
    } else {
#pragma unroll
      for (int s = 0; s < NV; ++s)
#pragma unroll
        for (int j = 0; j < 8; ++j) x[s][j] += y[s][j];
    }
  }
  const bool keep = !A.rows && b < n;
  auto store = [&](float* p, const float (&v)[8]) { __builtin_memcpy(__builtin_assume_aligned(p, 32), v, 32); };
  if (A.mix) {
    float* hr = A.hist + (size_t)t * D;
    const float a0 = A.mix[0], an = A.mix[A.n_hist];
#pragma unroll
    for (int s = 0; s < NV; ++s) {
      if (keep && at(s) < D) store(hr + (A.n_hist - 1) * A.hist_step + at(s), x[s]);
      float e[8];
      load(er + in(s), e);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[s][j] = a0 * e[j] + an * x[s][j];
    }
#pragma unroll 4
    for (int k = 1; k < A.n_hist; ++k) {
      const float ak = A.mix[k];
#pragma unroll
      for (int s = 0; s < NV; ++s) {
        float v[8];
        load(hr + (k - 1) * A.hist_step + in(s), v);
#pragma unroll
        for (int j = 0; j < 8; ++j) x[s][j] = fmaf(ak, v[j], x[s][j]);
      }
    }
  } else if (er) {
#pragma unroll
    for (int s = 0; s < NV; ++s) {
      float e[8];
      load(er + in(s), e);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[s][j] += e[j];
    }
  }
  if (keep && (A.y || er)) {
#pragma unroll
    for (int s = 0; s < NV; ++s)
      if (at(s) < D) store(rr + at(s), x[s]);
  }
  if (!A.out) return;  // (all of them)
  if (A.w_next) {
#pragma unroll
    for (int s = 0; s < NV; ++s) {
      ss[s] = 0.f;
#pragma unroll
      for (int j = 0; j < 8; ++j) ss[s] = fmaf(x[s][j], x[s][j], ss[s]);
      if (at(s) >= D) ss[s] = 0.f;
    }
    factors(ss, A.next_groups, inv);
  }
  if (b >= n) return;
  T* o = (T*)A.out + (size_t)b * A.ldo;
#pragma unroll
  for (int s = 0; s < NV; ++s) {
    if (at(s) >= A.ldo) continue;
    T a[8];
    float g[8];
    if (A.w_next && at(s) < D) load(A.w_next + at(s), g);
#pragma unroll
    for (int j = 0; j < 8; ++j) a[j] = (T)(at(s) >= D ? 0.f : A.w_next ? x[s][j] * inv[s] * g[j] : x[s][j]);
    __builtin_memcpy(__builtin_assume_aligned(o + at(s), sizeof(a)), a, sizeof(a));
  }
  for (int i = W * NV * 512 + (w * 64 + lane); i < A.ldo; i += 64 * W) o[i] = (T)0.f;
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
  // whole 8s, and groups that are lanes of a wave (a power of two) or whole wave steps
  auto lanes = [&](int g) { const int len = D / g, l = len / 8; return g == 1 || len % 512 == 0 || (len % 8 == 0 && l <= 64 && (l & (l - 1)) == 0); };
  const int steps = (D + 511) / 512;
  if (D % 8 == 0 && ldy % 8 == 0 && ldo % 8 == 0 && lanes(post_groups) && lanes(next_groups) && steps <= 16) {
    // many rows: as few waves a row as hold it in 4 vectors a thread; few: 4 waves
    const int w = n >= 1024 ? (steps <= 4 ? 1 : steps <= 8 ? 2 : 4) : 4, nv = (steps + w - 1) / w;
#define PA_RW(T, W, N) hipLaunchKernelGGL((residual_norm_wave_kernel<T, W, N>), dim3((n + 4 / W - 1) / (4 / W)), dim3(256), 0, st, A, n)
#define PA_RW_N(T, W)                       \
  do {                                      \
    if (nv == 1) PA_RW(T, W, 1);            \
    else if (nv == 2) PA_RW(T, W, 2);       \
    else PA_RW(T, W, 4);                    \
  } while (0)
#define PA_RW_T(T) do { if (w == 1) PA_RW_N(T, 1); else if (w == 2) PA_RW(T, 2, 4); else PA_RW_N(T, 4); } while (0)
    if (fp32) PA_RW_T(float); else PA_RW_T(pa::bf16);
#undef PA_RW_T
#undef PA_RW_N
#undef PA_RW
    return (int)hipGetLastError();
  }
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
