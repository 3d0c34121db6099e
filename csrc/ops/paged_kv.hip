// From a [q | k | v] projection row to the attention kernel's operands (window_attention.hip), in one
// launch: biases, RMS norms of heads, the rotation of the first rd dimensions of every query and key head (rd 0:
// none), queries to q_out, keys and values to their pages, and, where a token ends a block of `pool` tokens, the
// block's mean key and value.
//
//   x [T, ldx]    H x DK queries | G x DK keys | GV x DV values, bias likewise; the values may lie elsewhere in the
//                 row (at vcol), for instance on the keys: a value head is then a key head as projected
//   norms         per query and key head with a weight, per value head without one, over the real dimensions
//   pages         [pages, G, D/8, 16, 8]; pooled rows [pages, npb, G, D] with the page of the block's
//                 last token, blocks that end in one page in order
//
// A block's mean is taken over its rows as the cache holds them (rotated, in T). Small steps do it in the
// same launch: rows of earlier steps are read from their pages, rows of this step are computed again from
// the projection, so nothing waits for another workgroup. Larger steps have a second launch that reads
// all of them from their pages. Workgroups are dealt so that neighbouring tokens, which share the cache lines
// of a page, run on one XCD. Arithmetic is fp32.
#include "common.h"

namespace pa {
namespace kv {

struct Args {
  const void* x;
  const float* bias;  // optional
  void *q, *kp, *vp, *pk, *pv;
  const int *positions, *slots, *q_start, *q_len, *ctx_len, *block_table;
  const float* cos_sin;  // [max_pos, rd]: cos | sin
  const float *qn, *kn;  // norm weights [DK]; null: no norm of queries and keys
  int ldx, H, G, GV, DK, DV, rd, pool, npb, max_blocks, max_seqs, T;
  int vcol, norm_v;
  float ick, icv;  // 8 / DK, 8 / DV
  float idim, ivdim, eps;  // 1 / real dimensions
};

// u / n for the small numbers of here, with inv = 1 / n
__device__ __forceinline__ int quot(int u, float inv) { return (int)(((float)u + 0.5f) * inv); }

__device__ __forceinline__ void load8(const float* p, float (&v)[8]) {
  __builtin_memcpy(v, __builtin_assume_aligned(p, 16), 32);
}

// token of a workgroup: each of the 8 XCDs (workgroups go round) gets a contiguous eighth; -1: none
__device__ __forceinline__ int token_of(int b, int T) {
  const int per = (T + 7) >> 3, t = (b & 7) * per + (b >> 3);
  return (b >> 3) < per && t < T ? t : -1;
}

// the step's sequence that token t belongs to; every thread of the workgroup calls it
__device__ __forceinline__ int seq_of(const Args& A, int t, int* shared) {
  for (int i = threadIdx.x; i < A.max_seqs; i += 256) {
    const int q0 = A.q_start[i];
    if (q0 <= t && t < q0 + A.q_len[i]) *shared = i;
  }
  __syncthreads();
  return *shared;
}

// 8 values of head part `off` (columns off .. off + D of a row) from dimension d: biased, times inv * w (NORM), rotated
// by cs if `rot`
template <typename T, bool NORM>
__device__ __forceinline__ void chunk(const Args& A, const T* row, int off, int d, const float* cs, bool rot, float (&v)[8],
                                      float inv = 1.f, const float* w = nullptr) {
  const int half = A.rd >> 1;
  T a[8];
  __builtin_memcpy(a, __builtin_assume_aligned(row + off + d, sizeof(T) * 8), sizeof(T) * 8);
#pragma unroll
  for (int j = 0; j < 8; ++j) v[j] = (float)a[j];
  float b[8];
  if (A.bias) {
    load8(A.bias + off + d, b);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] += b[j];
  }
  if constexpr (NORM) {
    if (w) load8(w + d, b);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] *= w ? inv * b[j] : inv;
  }
  if (!rot || d >= A.rd) return;
  if (half % 8 == 0) {
    const int pd = d < half ? d + half : d - half, i = d < half ? d : d - half;
    __builtin_memcpy(a, __builtin_assume_aligned(row + off + pd, sizeof(T) * 8), sizeof(T) * 8);
    float c[8], s[8], u[8];
    load8(cs + i, c);
    load8(cs + half + i, s);
#pragma unroll
    for (int j = 0; j < 8; ++j) u[j] = (float)a[j];
    if (A.bias) {
      load8(A.bias + off + pd, b);
#pragma unroll
      for (int j = 0; j < 8; ++j) u[j] += b[j];
    }
    if constexpr (NORM) {
      if (w) load8(w + pd, b);
#pragma unroll
      for (int j = 0; j < 8; ++j) u[j] *= w ? inv * b[j] : inv;
    }
    const float sign = d < half ? -1.f : 1.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = v[j] * c[j] + sign * u[j] * s[j];
    return;
  }
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    const int e = d + j;
    if (e >= A.rd) break;
    const int pd = e < half ? e + half : e - half, i = e < half ? e : e - half;
    float u = (float)row[off + pd] + (A.bias ? A.bias[off + pd] : 0.f);
    if constexpr (NORM) u *= w ? inv * w[pd] : inv;
    v[j] = e < half ? v[j] * cs[i] - u * cs[half + i] : v[j] * cs[i] + u * cs[half + i];
  }
}

template <typename T>
__device__ __forceinline__ void put(T* dst, const float (&v)[8]) {
  T a[8];
#pragma unroll
  for (int j = 0; j < 8; ++j) a[j] = (T)v[j];
  __builtin_memcpy(__builtin_assume_aligned(dst, sizeof(T) * 8), a, sizeof(T) * 8);
}

// POOL: blocks that end here are pooled in this launch
template <typename T, bool POOL>
__global__ __launch_bounds__(256) void paged_kv_kernel(const Args A) {
  const int t = token_of(blockIdx.x, A.T);
  if (t < 0) return;
  const int slot = A.slots[t], pos = A.positions[t];
  if (slot < 0) return;
  const T* row = (const T*)A.x + (size_t)t * A.ldx;
  const float* cs = A.cos_sin + (size_t)pos * A.rd;
  const int ck = A.DK >> 3, cv = A.DV >> 3, nq = A.H * ck, nk = A.G * ck, nv = A.GV * cv;
  for (int u = threadIdx.x; u < nq + nk + nv; u += 256) {
    float v[8];
    if (u < nq) {
      const int h = quot(u, A.ick), d = (u - h * ck) * 8;
      chunk<T, false>(A, row, h * A.DK, d, cs, true, v);
      put((T*)A.q + ((size_t)t * A.H + h) * A.DK + d, v);
    } else {
      const bool key = u < nq + nk;
      const int w = key ? u - nq : u - nq - nk, per = key ? ck : cv, D = key ? A.DK : A.DV;
      const int h = quot(w, key ? A.ick : A.icv), o = w - h * per;
      chunk<T, false>(A, row, (key ? A.H * A.DK : A.vcol) + h * D, o * 8, cs, key, v);
      put((T*)(key ? A.kp : A.vp) + (((size_t)(slot >> 4) * (key ? A.G : A.GV) + h) * per + o) * 128 + (slot & 15) * 8, v);
    }
  }
  if constexpr (!POOL) return;
  const int P = A.pool;
  if ((pos + 1) % P) return;
  __shared__ int seq;
  const int lo = seq_of(A, t, &seq);
  const int start = A.ctx_len[lo] - A.q_len[lo];  // the step's first position
  const int* bt = A.block_table + (size_t)lo * A.max_blocks;
  const int page = pos >> 4, sub = pos / P - (page << 4) / P;
  const float inv = 1.f / (float)P;
  for (int u = threadIdx.x; u < nk + nv; u += 256) {
    const bool key = u < nk;
    const int w = key ? u : u - nk, per = key ? ck : cv, D = key ? A.DK : A.DV;
    const int h = w / per, o = w - h * per, off = (key ? A.H * A.DK : A.vcol) + h * D;
    float sum[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int p = pos - P + 1; p <= pos; ++p) {
      if (p < start) {
        T a[8];
        const T* src = (const T*)(key ? A.kp : A.vp) + (((size_t)bt[p >> 4] * A.G + h) * per + o) * 128 + (p & 15) * 8;
        __builtin_memcpy(a, __builtin_assume_aligned(src, sizeof(T) * 8), sizeof(T) * 8);
#pragma unroll
        for (int j = 0; j < 8; ++j) sum[j] += (float)a[j];
      } else {
        float v[8];
        chunk<T, false>(A, row - (size_t)(pos - p) * A.ldx, off, o * 8, A.cos_sin + (size_t)p * A.rd, key, v);
#pragma unroll
        for (int j = 0; j < 8; ++j) sum[j] += (float)(T)v[j];
      }
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) sum[j] *= inv;
    put((T*)(key ? A.pk : A.pv) + (((size_t)(slot >> 4) * A.npb + sub) * A.G + h) * D + o * 8, sum);
  }
}

// lanes of a head of D dimensions, as a power of two
__host__ __device__ __forceinline__ int head_bits(int D) {
  int b = 0;
  while ((8 << b) < D) ++b;
  return b;
}
// units of 8 dimensions: queries and keys, then, from a whole wave on, values
__host__ __device__ __forceinline__ int normed_units(int heads, int values, int DK, int DV, int* nqk) {
  *nqk = ((heads << head_bits(DK)) + 63) & ~63;
  return *nqk + (values << head_bits(DV));
}

// With norms: a power of two of lanes per head, which sum its squares. A unit's loads go out together.
template <typename T>
__global__ __launch_bounds__(512) void normed_kv_kernel(const Args A) {
  const int t = token_of(blockIdx.x, A.T);
  if (t < 0) return;
  const int slot = A.slots[t], pos = A.positions[t];
  if (slot < 0) return;
  const T* row = (const T*)A.x + (size_t)t * A.ldx;
  const float* cs = A.cos_sin + (size_t)pos * A.rd;
  const int ck = A.DK >> 3, cv = A.DV >> 3, half = A.rd >> 1;
  const int bk = head_bits(A.DK), bv = head_bits(A.DV);
  int nqk;
  const int total = normed_units(A.H + A.G, A.GV, A.DK, A.DV, &nqk);
  for (int u0 = 0; u0 < total; u0 += blockDim.x) {
    const int u = u0 + threadIdx.x;
    const bool value = u >= nqk;
    const int w = value ? u - nqk : u, bits = value ? bv : bk, per = value ? cv : ck;
    const int h = w >> bits, d = (w & ((1 << bits) - 1)) * 8;  // (query heads, then key heads)
    const bool in = d < per * 8 && h < (value ? A.GV : A.H + A.G), query = !value && h < A.H;
    const int off = value ? A.vcol + h * A.DV : h * A.DK;
    const float* nw = value ? nullptr : query ? A.qn : A.kn;
    const bool normed = value ? A.norm_v != 0 : nw != nullptr;
    const bool turn = in && !value && d < A.rd, whole = half % 8 == 0;
    const int pd = d < half ? d + half : d - half, ci = d < half ? d : pd;
    float v[8], p[8], c[8], s[8], wv[8], wp[8], ss = 0.f;
    if (in) {
      chunk<T, false>(A, row, off, d, cs, false, v);
      if (nw) load8(nw + d, wv);
      if (turn && whole) {
        chunk<T, false>(A, row, off, pd, cs, false, p);
        if (nw) load8(nw + pd, wp);
        load8(cs + ci, c);
        load8(cs + half + ci, s);
      }
#pragma unroll
      for (int j = 0; j < 8; ++j) ss = fmaf(v[j], v[j], ss);
    }
    for (int m = (1 << bits) >> 1; m > 0; m >>= 1) ss += __shfl_xor(ss, m, 64);
    if (!in) continue;
    const float inv = normed ? 1.f / sqrtf(ss * (value ? A.ivdim : A.idim) + A.eps) : 1.f;
    if (turn && !whole) {
      chunk<T, true>(A, row, off, d, cs, true, v, inv, nw);
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] *= nw ? inv * wv[j] : inv;
      if (turn) {
        const float sign = d < half ? -inv : inv;
#pragma unroll
        for (int j = 0; j < 8; ++j) v[j] = v[j] * c[j] + sign * (nw ? p[j] * wp[j] : p[j]) * s[j];
      }
    }
    if (query) {
      put((T*)A.q + ((size_t)t * A.H + h) * A.DK + d, v);
    } else {
      const int g = value ? h : h - A.H;
      put((T*)(value ? A.vp : A.kp) + (((size_t)(slot >> 4) * (value ? A.GV : A.G) + g) * per + (d >> 3)) * 128 + (slot & 15) * 8, v);
    }
  }
}

// The blocks that end in this step, from their pages: a workgroup per `rows` tokens.
template <typename T>
__global__ __launch_bounds__(256) void pool_kernel(const Args A, int rows) {
  __shared__ int seq;
  const int P = A.pool, ck = A.DK >> 3, cv = A.DV >> 3, nk = A.G * ck, nv = A.G * cv;
  const float inv = 1.f / (float)P;
  const int end = min(A.T, ((int)blockIdx.x + 1) * rows);
  for (int t = blockIdx.x * rows; t < end; ++t) {
    const int slot = A.slots[t], pos = A.positions[t];
    if (slot < 0 || (pos + 1) % P) continue;
    __syncthreads();
    const int* bt = A.block_table + (size_t)seq_of(A, t, &seq) * A.max_blocks;
    const int page = pos >> 4, sub = pos / P - (page << 4) / P;
    for (int u = threadIdx.x; u < nk + nv; u += 256) {
      const bool key = u < nk;
      const int w = key ? u : u - nk, per = key ? ck : cv, D = key ? A.DK : A.DV;
      const int h = quot(w, key ? A.ick : A.icv), o = w - h * per;
      float sum[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
      for (int p = pos - P + 1; p <= pos; ++p) {
        T a[8];
        const T* src = (const T*)(key ? A.kp : A.vp) + (((size_t)bt[p >> 4] * A.G + h) * per + o) * 128 + (p & 15) * 8;
        __builtin_memcpy(a, __builtin_assume_aligned(src, sizeof(T) * 8), sizeof(T) * 8);
#pragma unroll
        for (int j = 0; j < 8; ++j) sum[j] += (float)a[j];
      }
#pragma unroll
      for (int j = 0; j < 8; ++j) sum[j] *= inv;
      put((T*)(key ? A.pk : A.pv) + (((size_t)(slot >> 4) * A.npb + sub) * A.G + h) * D + o * 8, sum);
    }
  }
}

}  // namespace kv
}  // namespace pa

extern "C" int pa_paged_kv(int fp32, const void* x, const float* bias, void* q, void* kp, void* vp, void* pk, void* pv,
                           const int* positions, const int* slots, const int* q_start, const int* q_len,
                           const int* ctx_len, const int* block_table, const float* cos_sin, int ldx, int H, int G, int GV,
                           int DK, int DV, int rd, int pool, int npb, int max_blocks, int max_seqs, int T, int vcol,
                           const float* qn, const float* kn, int norm_v, int dim, int vdim, float eps, hipStream_t st) {
  if (T <= 0) return 0;
  const bool normed = qn || kn || norm_v;
  if (DK % 8 || DV % 8 || rd % 2 || rd > DK || ldx % 8 || vcol % 8 || (pool > 0 && (normed || G != GV))) return -1;
  if (normed && (DK > 512 || DV > 512 || dim <= 0 || vdim <= 0)) return -2;  // a head in a wave
  const pa::kv::Args A{x, bias, q, kp, vp, pk, pv, positions, slots, q_start, q_len, ctx_len, block_table, cos_sin, qn, kn,
                       ldx, H, G, GV, DK, DV, rd, pool, npb, max_blocks, max_seqs, T, vcol, norm_v, 8.f / DK, 8.f / DV,
                       normed ? 1.f / dim : 0.f, normed ? 1.f / vdim : 0.f, eps};
  const dim3 grid((T + 7) / 8 * 8);
  if (normed) {
    int nqk;
    const int total = pa::kv::normed_units(H + G, GV, DK, DV, &nqk), rounds = (total + 511) / 512;
    const dim3 wg(((total + rounds - 1) / rounds + 63) / 64 * 64);
    if (fp32) hipLaunchKernelGGL(pa::kv::normed_kv_kernel<float>, grid, wg, 0, st, A);
    else hipLaunchKernelGGL(pa::kv::normed_kv_kernel<pa::bf16>, grid, wg, 0, st, A);
    return (int)hipGetLastError();
  }
  const bool later = pool > 0 && T > 64, now = pool > 0 && !later;
  const int rows = pool < 8 ? pool : 8;  // of a workgroup of the second launch
#define PA_KV(TYPE)                                                                                              \
  do {                                                                                                           \
    if (now) hipLaunchKernelGGL((pa::kv::paged_kv_kernel<TYPE, true>), grid, dim3(256), 0, st, A);               \
    else hipLaunchKernelGGL((pa::kv::paged_kv_kernel<TYPE, false>), grid, dim3(256), 0, st, A);                  \
    if (later) hipLaunchKernelGGL(pa::kv::pool_kernel<TYPE>, dim3((T + rows - 1) / rows), dim3(256), 0, st, A, rows); \
  } while (0)
  if (fp32) PA_KV(float); else PA_KV(pa::bf16);
#undef PA_KV
  return (int)hipGetLastError();
}
