// Routing by score: which experts a token uses, with what weights, and the rows of all tokens sorted
// by expert for the grouped projections (grouped_gemm.hip).
//
//   z = W_router h (fp32 sums; h and W in T),  s = sigmoid(z), or softmax(z) over all experts
//   c = s + correction (if there is one)
//   group's score = the sum of its two largest c; the `keep` best of `groups` equal groups of neighbours stay
//   the `top` experts with the largest c among them are chosen, with weights scale * s, or with `share`
//   scale * s / (sum of the chosen s + 1e-20)
//   `always` more experts (numbers E .. E + always - 1) follow for every token, with weight 1
//
// Ties go to the lower number. One workgroup scores 16 tokens. Steps of at most 16 tokens sort in the
// same launch; otherwise a workgroup takes its rows' places within every expert from global
// counters (their order has no meaning) and place_kernel, a second launch, turns them into positions.
// Rows with slot < 0 (padding) are left out.
#include "common.h"

#include <algorithm>
#include <climits>

namespace pa {
namespace sr {

constexpr int TOK = 16, NT = 512, MAX_E = 1024;

struct Args {
  const void* h;      // [T, ldh]
  const void* w;      // bf16: packed [E/16, K/32, 64, 8]; fp32: [E, K]
  const int* slots;
  float* weights;     // [T, top + always]
  int *choice, *rank; // [T, top + always]
  int* counts;        // [E + always], zero before the launch (unused with one workgroup)
  int* order;         // position -> token * (top + always) + k
  int4* tiles;        // {expert, first position, rows, 0}
  int* n_tiles;
  const float* correction;  // [E] or null
  int T, ldh, K, E, top, groups, keep, always, tm, max_tiles;
  int softmax, share;
  float scale;
};

// floats and integers in the same order, with room at both ends whatever the bits are
__device__ __forceinline__ int ordered(float v) {
  const int i = __float_as_int(v);
  return min(max(i ^ ((i >> 31) & 0x7fffffff), INT_MIN + 2), INT_MAX - 1);
}

// Exclusive sums of cnt over experts into base (rows) and tbase (tiles of tm rows); returns the tiles.
// All NT threads call it; cnt, base, tbase are in LDS.
__device__ __forceinline__ int scan_counts(const int* cnt, int* base, int* tbase, int E, int tm, int (*ws)[NT / 64]) {
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  int carry_r = 0, carry_t = 0;
  for (int e0 = 0; e0 < E; e0 += NT) {
    const int e = e0 + threadIdx.x;
    const int r = e < E ? cnt[e] : 0, q = (r + tm - 1) / tm;
    int sr = r, sq = q;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int a = __shfl_up(sr, o, 64), b = __shfl_up(sq, o, 64);
      if (lane >= o) { sr += a; sq += b; }
    }
    if (lane == 63) { ws[0][wid] = sr; ws[1][wid] = sq; }
    __syncthreads();
    int br = carry_r, bq = carry_t, tr = 0, tq = 0;
    for (int w = 0; w < NT / 64; ++w) {
      if (w < wid) { br += ws[0][w]; bq += ws[1][w]; }
      tr += ws[0][w];
      tq += ws[1][w];
    }
    if (e < E) { base[e] = br + sr - r; tbase[e] = bq + sq - q; }
    carry_r += tr;
    carry_t += tq;
    __syncthreads();
  }
  return carry_t;
}

__device__ __forceinline__ void write_tiles(const Args& A, const int* cnt, const int* base, const int* tbase, int E, int n) {
  for (int e = threadIdx.x; e < E; e += NT)
    for (int i = 0, k = tbase[e]; i < cnt[e]; i += A.tm, ++k)
      if (k < A.max_tiles) A.tiles[k] = int4{e, base[e] + i, min(A.tm, cnt[e] - i), 0};
  if (threadIdx.x == 0) A.n_tiles[0] = min(n, A.max_tiles);
}

template <typename T>
__global__ __launch_bounds__(NT) void score_kernel(const Args A) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int Ep = (A.E + 15) / 16 * 16, EA = A.E + A.always;
  float* sc = sm;                       // [TOK][Ep] scores
  float* gs = sc + TOK * Ep;            // [TOK][groups]
  float* sel = gs + TOK * A.groups;     // [TOK][top] scores of the chosen
  float* red = sel + TOK * A.top;       // bf16: [8][16][64 + 4]; then [TOK][Ep], what the choice goes by
  int* cnt = (int*)(red + max(8 * 16 * 68, TOK * Ep)); // [EA], then base, tbase
  int *base = cnt + EA, *tbase = base + EA;
  __shared__ int ws[2][NT / 64];
  const int t0 = blockIdx.x * TOK, lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  for (int e = threadIdx.x; e < EA; e += NT) cnt[e] = 0;
  if constexpr (sizeof(T) == 2) {
    // 8 waves over K, 64 experts at a time: D = W . h^T, a lane holds 4 experts of one token
    const int g = lane >> 4, c = lane & 15, K32 = A.K / 32, tiles = Ep / 16;
    const bf16* hr = (const bf16*)A.h + (size_t)min(t0 + c, A.T - 1) * A.ldh + 8 * g;
    for (int e0 = 0; e0 < tiles; e0 += 4) {
      f32x4 acc[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
      const bf16* wt[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) wt[i] = (const bf16*)A.w + (size_t)min(e0 + i, tiles - 1) * K32 * 512 + lane * 8;
#pragma unroll 8
      for (int k = wid; k < K32; k += 8) {
        const bf16x8 b = *reinterpret_cast<const bf16x8*>(hr + 32 * k);
#pragma unroll
        for (int i = 0; i < 4; ++i)
          acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(wt[i] + (size_t)k * 512), b, acc[i], 0, 0, 0);
      }
      __syncthreads();
#pragma unroll
      for (int i = 0; i < 4; ++i) *reinterpret_cast<f32x4*>(red + (wid * 16 + c) * 68 + 16 * i + 4 * g) = acc[i];
      __syncthreads();
      for (int p = threadIdx.x; p < 16 * 64; p += NT) {
        const int t = p >> 6, e = p & 63;
        float z = 0.f;
#pragma unroll
        for (int w = 0; w < 8; ++w) z += red[(w * 16 + t) * 68 + e];
        if (e0 * 16 + e < Ep) sc[t * Ep + e0 * 16 + e] = A.softmax ? z : 1.f / (1.f + expf(-z));
      }
    }
  } else {
    for (int p = threadIdx.x; p < TOK * A.E; p += NT) {
      const int t = p / A.E, e = p - t * A.E;
      const float *x = (const float*)A.h + (size_t)min(t0 + t, A.T - 1) * A.ldh, *w = (const float*)A.w + (size_t)e * A.K;
      float z[4] = {0.f, 0.f, 0.f, 0.f};
      for (int k = 0; k < A.K; k += 4)
#pragma unroll
        for (int j = 0; j < 4; ++j) z[j] = fmaf(x[k + j], w[k + j], z[j]);
      const float v = (z[0] + z[1]) + (z[2] + z[3]);
      sc[t * Ep + e] = A.softmax ? v : 1.f / (1.f + expf(-v));
    }
  }
  __syncthreads();
  // 32 lanes per token. Nothing is chosen one after the other: a group, or an expert, is in when fewer than
  // `keep`, or `top`, others come before it (larger, or equal and lower), and that number is its place.
  // Scores are compared as integers in the floats' order, and no two are alike in rank whatever the bits are.
  const int tk = threadIdx.x >> 5, l = threadIdx.x & 31, t = t0 + tk, KA = A.top + A.always;
  const bool live = t < A.T && A.slots[min(t, A.T - 1)] >= 0;
  float *s = sc + tk * Ep, *gr = gs + tk * A.groups, *se = sel + tk * A.top;
  float* cf = red + tk * Ep;
  int *si = (int*)cf, *gi = (int*)gr;
  constexpr int OUT = INT_MIN + 1, PAD = INT_MIN;
  if (A.softmax) {
    float m = -INFINITY, sum = 0.f;
    for (int e = l; e < A.E; e += 32) m = fmaxf(m, s[e]);
#pragma unroll
    for (int o = 16; o > 0; o >>= 1) m = fmaxf(m, __shfl_xor(m, o, 64));
    for (int e = l; e < A.E; e += 32) {
      const float p = expf(s[e] - m);
      s[e] = p;
      sum += p;
    }
#pragma unroll
    for (int o = 16; o > 0; o >>= 1) sum += __shfl_xor(sum, o, 64);
    const float inv = 1.f / sum;
    for (int e = l; e < A.E; e += 32) s[e] *= inv;
  }
  for (int e = l; e < A.E; e += 32) cf[e] = A.correction ? s[e] + A.correction[e] : s[e];
  __syncthreads();
  if (A.keep < A.groups) {
    const int per = A.E / A.groups;
    for (int i = l; i < A.groups; i += 32) {
      float a = -INFINITY, b = -INFINITY;
#pragma unroll 4
      for (int e = i * per; e < (i + 1) * per; ++e) {
        const float v = cf[e];
        b = fmaxf(b, fminf(a, v));
        a = fmaxf(a, v);
      }
      gi[i] = ordered(a + (per > 1 ? b : 0.f));
    }
    __syncthreads();
  }
  for (int e = l; e < Ep; e += 32) si[e] = e < A.E ? ordered(cf[e]) : PAD;
  __syncthreads();
  if (A.keep < A.groups) {
    const int per = A.E / A.groups;
    for (int i = l; i < A.groups; i += 32) {
      int before = 0;
      const int v = gi[i];
#pragma unroll 4
      for (int k = 0; k < A.groups; ++k) before += gi[k] > v || (gi[k] == v && k < i);
      if (before >= A.keep)
        for (int e = i * per; e < (i + 1) * per; ++e) si[e] = OUT;
    }
    __syncthreads();
  }
  float chosen = 0.f;
  for (int e0 = l; e0 < A.E; e0 += 64) {  // two experts a lane
    const int ea = e0, eb = min(e0 + 32, Ep - 1), va = si[ea], vb = si[eb];
    int na = 0, nb = 0;
#pragma unroll 4
    for (int k = 0; k < Ep; k += 4) {
      const int4 q = *reinterpret_cast<const int4*>(si + k);
      const int w[4] = {q.x, q.y, q.z, q.w};
#pragma unroll
      for (int j = 0; j < 4; ++j) {  // an equal score with a lower number comes first
        na += w[j] >= va + (k + j >= ea);
        nb += w[j] >= vb + (k + j >= eb);
      }
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int e = i ? e0 + 32 : e0, before = i ? nb : na;
      if (e < A.E && before < A.top && live) {
        A.choice[(size_t)t * KA + before] = e;
        se[before] = s[e];
        chosen += s[e];
        A.rank[(size_t)t * KA + before] = atomicAdd(&cnt[e], 1);
      }
    }
  }
  if (t < A.T && !live)  // (a row of padding holds anything)
    for (int i = l; i < A.top; i += 32) A.choice[(size_t)t * KA + i] = -1;
#pragma unroll
  for (int o = 16; o > 0; o >>= 1) chosen += __shfl_xor(chosen, o, 64);
  const float f = A.share ? A.scale / (chosen + 1e-20f) : A.scale;
  __syncthreads();
  if (t < A.T)
    for (int i = l; i < A.top; i += 32) A.weights[(size_t)t * KA + i] = live ? se[i] * f : 0.f;
  if (l < A.always && t < A.T) {
    const size_t p = (size_t)t * KA + A.top + l;
    A.choice[p] = live ? A.E + l : -1;
    A.weights[p] = live ? 1.f : 0.f;
    if (live) A.rank[p] = atomicAdd(&cnt[A.E + l], 1);
  }
  __syncthreads();
  if (gridDim.x == 1) {
    const int n = scan_counts(cnt, base, tbase, EA, A.tm, ws);
    write_tiles(A, cnt, base, tbase, EA, n);
    for (int p = threadIdx.x; p < A.T * KA; p += NT) {  // (this workgroup's own writes, behind its barriers)
      const int e = A.choice[p];
      if (e >= 0) A.order[base[e] + A.rank[p]] = p;
    }
    return;
  }
  for (int e = threadIdx.x; e < EA; e += NT)
    if (cnt[e]) base[e] = atomicAdd(&A.counts[e], cnt[e]);
  __syncthreads();
  for (int p = t0 * KA + threadIdx.x; p < min(t0 + TOK, A.T) * KA; p += NT) {
    const int e = A.choice[p];
    if (e >= 0) A.rank[p] += base[e];
  }
}

__global__ __launch_bounds__(NT) void place_kernel(const Args A) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ int ws[2][NT / 64];
  const int EA = A.E + A.always, P = A.T * (A.top + A.always);
  int *cnt = (int*)sm, *base = cnt + EA, *tbase = base + EA;
  for (int e = threadIdx.x; e < EA; e += NT) cnt[e] = A.counts[e];
  __syncthreads();
  const int n = scan_counts(cnt, base, tbase, EA, A.tm, ws);
  if (blockIdx.x == 0) write_tiles(A, cnt, base, tbase, EA, n);
  for (int p = blockIdx.x * NT + threadIdx.x; p < P; p += gridDim.x * NT) {
    const int e = A.choice[p];
    if (e >= 0) A.order[base[e] + A.rank[p]] = p;
  }
}

}  // namespace sr
}  // namespace pa

extern "C" int pa_score_route(int fp32, const void* h, int ldh, const void* w, int K, const int* slots, float* weights,
                              int* choice, int* rank, int* counts, int* order, int* tiles, int* n_tiles, int T, int E,
                              int top, int groups, int keep, int always, int tm, int max_tiles, int softmax,
                              const float* correction, int share, float scale, hipStream_t st) {
  using namespace pa::sr;
  if (T <= 0) return 0;
  if (E < 1 || E + always > MAX_E || always > 32 || groups < 1 || E % groups || keep < 1 || keep > groups || top < 1 ||
      top > keep * (E / groups) || K % 32 || ldh % 8) return -1;
  const Args A{h, w, slots, weights, choice, rank, counts, order, (int4*)tiles, n_tiles, correction, T, ldh, K, E, top, groups,
               keep, always, tm, max_tiles, softmax, share, scale};
  const int Ep = (E + 15) / 16 * 16, lds = (TOK * (Ep + groups + top) + 3 * (E + always) + std::max(8 * 16 * 68, TOK * Ep) + 64) * 4;
  static bool attr = false;
  if (!attr) {
    (void)hipFuncSetAttribute((const void*)score_kernel<float>, hipFuncAttributeMaxDynamicSharedMemorySize, 159 * 1024);
    (void)hipFuncSetAttribute((const void*)score_kernel<pa::bf16>, hipFuncAttributeMaxDynamicSharedMemorySize, 159 * 1024);
    attr = true;
  }
  if (lds > 159 * 1024) return -2;
  const int wgs = (T + TOK - 1) / TOK;
  if (fp32) hipLaunchKernelGGL(score_kernel<float>, dim3(wgs), dim3(NT), lds, st, A);
  else hipLaunchKernelGGL(score_kernel<pa::bf16>, dim3(wgs), dim3(NT), lds, st, A);
  if (wgs > 1)
    hipLaunchKernelGGL(place_kernel, dim3(std::min(256, (T * (top + always) + NT - 1) / NT)), dim3(NT),
                       3 * (E + always) * 4, st, A);
  return (int)hipGetLastError();
}
