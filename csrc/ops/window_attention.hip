// Paged grouped-query attention with a sliding window or chunks, kept first tokens, pooled keys before the window,
// capped scores, a bias by distance, a sink in the softmax's denominator and an output gate, for prefill chunks,
// decode rows and mixed batches in one launch.
//
//   position i sees   keys j <= i with i - j < W or j < keep (W 0: every j <= i), or those of its chunk of C
//                     positions (C > 0: j >= i - i % C), and, with P > 0,
//                     block b (the mean key and value of positions bP .. bP + P - 1) if
//                     bP + P - 1 <= i - W, that is b < (i - W + 1) / P
//   s = cap tanh(q . k scale / cap) - slope_h (i - j)         (cap 0: no cap; no slopes: no bias)
//   out = gain sigmoid(gate) sum p v,   p = exp(s) / (exp(sink_h) + sum exp(s)), one softmax over all kinds
//
// R = H / G query heads share a key head, G / GV key heads a value head (differential attention: 2). Keys and values are fragment-major pages of 16 tokens per KV head, [D/8][16][8] (paged_kv.hip); the
// value operand of the second product comes from the same form by LDS transpose reads. A pooled
// block's row lies with the page of its last token: [page][per page][KV head][D]. 16 of them, gathered
// row by row, make a tile of the same form as a page, so both kinds of keys run the same code:
//
//   S^T[keys x cols] = K . Q^T         cols = (token, query head of the KV head's group) pairs
//   O^T[dims x cols] += V^T . P^T      P^T = the S^T accumulator's own registers
//
// An item's keys are its pooled blocks (a tile at a time), the tiles of the kept tokens that lie before its window's,
// and then the tiles of its window or chunk. Items
// come from the scheduler like paged_attention's (seq, q_begin, nq | part<<8 | nparts<<20, partial slot):
//   nq <= dec_tokens: split over keys. The 8 waves take every 8th page with a private LDS tile and merge;
//                     nparts > 1 divides the item's own key range, merge_kernel combines the partitions.
//   otherwise:        128 columns per workgroup, 16 per wave; all waves share double-buffered tiles of 64 keys
//                     (32 for the widest heads) that arrive by direct global -> LDS loads. Few such items are
//                     cut over keys too.
#include "common.h"

#include <algorithm>

namespace pa {
namespace wa {

constexpr float NEG_BIG = -1.0e30f;
typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) bf16x4 lds_bf16x4;
typedef __attribute__((address_space(3))) void lds_void;
typedef const __attribute__((address_space(1))) void glb_void;

struct Args {
  void* out;             // [T, ldo]: H x DV
  float* part_o;         // [G, slots, NB, 16, DV]
  float* part_ml;        // [G, slots, NB, 16, 2]
  const void* q;         // [T, H, DK]
  const void *kp, *vp;   // [pages, G, D/8, 16, 8]
  const void *pk, *pv;   // [pages, npb, G, D]
  const int4* items;
  const int* n_items;
  const int *q_start, *q_len, *ctx_len, *block_table;
  int max_blocks, max_items, H, G, R, NB, DK, DV, dec_tokens, window, pool, npb;
  float scale_log2;
  const float *sink, *slopes;  // [H] or null: log of the sink, bias per token of distance
  const void* gate;            // [T, ldg]: H x DV, or null
  float scale, cap, gain;
  int GV, keep, chunk, ldo, ldg, out_f32;
};

constexpr float LOG2E = 1.4426950408889634f;

__device__ __forceinline__ int first_key(const Args& A, int pos) {
  return A.window > 0 ? max(0, pos - A.window + 1) : A.chunk > 0 ? pos - pos % A.chunk : 0;
}
// tiles of `keys` kept tokens that lie before tile k_lo
__device__ __forceinline__ int kept_tiles(const Args& A, int keys, int k_lo) { return min((A.keep + keys - 1) / keys, k_lo); }
// pooled blocks that position pos sees
__device__ __forceinline__ int blocks_of(const Args& A, int pos) {
  return A.pool > 0 && A.window > 0 ? max(0, pos - A.window + 1) / A.pool : 0;
}
// row index of pooled block b of KV head h
__device__ __forceinline__ size_t pooled_row(const Args& A, const int* bt, int b, int h) {
  const int page = (b * A.pool + A.pool - 1) >> 4;
  return ((size_t)bt[page] * A.npb + (b - (page << 4) / A.pool)) * A.G + h;
}

// A score's cap and bias, in units of q . k, which the softmax's scale still multiplies. Within a tile the bias is
// slope * (key - first key) on the scores and -slope * (distance to the first key) on all of a lane's scores alike.
enum { NO_MODS = 0, CAP = 1, BIAS = 2 };  // BIAS: and a cap, if there is one

template <int MODS>
struct Mods {
  float to_tanh = 0.f, from_tanh = 0.f, slope = 0.f;
  __device__ __forceinline__ Mods(const Args& A, int head) {
    if (MODS != NO_MODS) {
      to_tanh = A.cap > 0.f ? 2.f * LOG2E * A.scale / A.cap : 0.f;
      from_tanh = A.cap / A.scale;
    }
    if (MODS == BIAS) slope = A.slopes[head] / A.scale;
  }
  __device__ __forceinline__ float capped(float s) const {  // from_tanh * tanh
    const float r = __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(s * to_tanh));
    return fmaf(r, -2.f * from_tanh, from_tanh);
  }
  template <int N>
  __device__ __forceinline__ void cap(f32x4 (&s)[N]) const {  // (one branch for all of them)
    if (MODS == CAP || (MODS == BIAS && to_tanh != 0.f)) {
#pragma unroll
      for (int k = 0; k < N; ++k)
#pragma unroll
        for (int r = 0; r < 4; ++r) s[k][r] = capped(s[k][r]);
    }
  }
};

// four outputs of head h at dimension d of a token's row, with gain and gate
template <typename T, int N>
__device__ __forceinline__ void put_out(const Args& A, size_t tok, int h, int d, float (&v)[N]) {
#pragma unroll
  for (int j = 0; j < N; ++j) v[j] *= A.gain;
  if (A.gate) {
    T g[N];
    __builtin_memcpy(g, __builtin_assume_aligned((const T*)A.gate + tok * A.ldg + (size_t)h * A.DV + d, sizeof(T) * N), sizeof(T) * N);
#pragma unroll
    for (int j = 0; j < N; ++j) v[j] /= 1.f + __expf(-(float)g[j]);
  }
  const size_t at = tok * A.ldo + (size_t)h * A.DV + d;
  if (A.out_f32) {
    __builtin_memcpy(__builtin_assume_aligned((float*)A.out + at, 4 * N), v, 4 * N);
  } else {
    T o[N];
#pragma unroll
    for (int j = 0; j < N; ++j) o[j] = (T)v[j];
    __builtin_memcpy(__builtin_assume_aligned((T*)A.out + at, sizeof(T) * N), o, sizeof(T) * N);
  }
}

// ---------------------------------------------------------------------------
// Any sizes, bf16 or fp32: one workgroup per (token of an item, head). The exact path.
template <typename T>
__global__ __launch_bounds__(256) void simple_kernel(const Args A) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float* sq = sm;            // DK
  float* sp = sm + A.DK;     // 256
  float* red = sp + 256;     // 4
  const int h = blockIdx.x, n = A.n_items[0], gk = h / A.R, gv = gk / (A.G / A.GV);
  const float slope = A.slopes ? A.slopes[h] * LOG2E : 0.f, sink = A.sink ? A.sink[h] * LOG2E : NEG_BIG;
  for (int item = blockIdx.y; item < n; item += gridDim.y) {
    const int4 it = A.items[item];
    const int s = it.x, nq = it.z & 0xff, part = (it.z >> 8) & 0xfff;
    if (part > 0) continue;  // partition 0 takes the whole range
    const int ctx = A.ctx_len[s], ql = A.q_len[s];
    const int* bt = A.block_table + (size_t)s * A.max_blocks;
    for (int i = 0; i < nq; ++i) {
      const int tok = it.y + i, pos = ctx - ql + tok;
      const int lo = first_key(A, pos), nb = blocks_of(A, pos), kept = min(A.keep, lo), front = nb + kept, total = front + pos - lo + 1;
      const size_t row = (size_t)(A.q_start[s] + tok) * A.H + h;
      // element d of key (or value) kk: pooled blocks first, then the kept and the window's tokens
      auto key_of = [&](int kk) { return kk < front ? kk - nb : lo + kk - front; };
      auto at = [&](const void* pages, const void* pooled, int heads, int g, int D, int kk, int d) -> float {
        if (kk < nb) return (float)((const T*)pooled)[pooled_row(A, bt, kk, g) * D + d];
        const int key = key_of(kk);
        return (float)((const T*)pages)[((size_t)bt[key >> 4] * heads + g) * D * 16 + (size_t)(d >> 3) * 128 + (key & 15) * 8 + (d & 7)];
      };
      __syncthreads();
      for (int d = threadIdx.x; d < A.DK; d += 256) sq[d] = (float)((const T*)A.q)[row * A.DK + d];
      __syncthreads();
      float m = sink, l = A.sink ? 1.f : 0.f, o[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
      for (int k0 = 0; k0 < total; k0 += 256) {
        const int kk = k0 + threadIdx.x;
        float sc = NEG_BIG;
        if (kk < total) {
          float a = 0.f;
          for (int d = 0; d < A.DK; ++d) a += sq[d] * at(A.kp, A.pk, A.G, gk, A.DK, kk, d);
          sc = a * A.scale_log2;
          if (A.cap > 0.f) sc = A.cap * LOG2E * tanhf(a * A.scale / A.cap);
          if (kk >= nb) sc -= slope * (float)(pos - key_of(kk));
        }
        const float wm = wave_max(sc);
        if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = wm;
        __syncthreads();
        const float mn = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
        const float alpha = exp2f(m - mn), p = kk < total ? exp2f(sc - mn) : 0.f;
        m = mn;
        sp[threadIdx.x] = p;
        __syncthreads();
        l = l * alpha + block_sum<4>(p, red);
        const int nk = min(256, total - k0);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const int d = threadIdx.x + 256 * e;
          if (d >= A.DV) break;
          float a = o[e] * alpha;
          for (int k = 0; k < nk; ++k) a += sp[k] * at(A.vp, A.pv, A.GV, gv, A.DV, k0 + k, d);
          o[e] = a;
        }
        __syncthreads();
      }
      const float inv = 1.f / l;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int d = threadIdx.x + 256 * e;
        float v[1] = {o[e] * inv};
        if (d < A.DV) put_out<T>(A, (size_t)(A.q_start[s] + tok), h, d, v);
      }
    }
  }
}

// ---------------------------------------------------------------------------
// V^T operand: lanes 16g + i of the result hold dim i of keys 4g .. 4g + 3; each lane names the
// 8 bytes (key 4g + i/4, dims 4 (i%4) .. + 3) of the 4 x 16 block its group transposes
__device__ __forceinline__ bf16x4 tr_read(const char* p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds_bf16x4*)p);
}

constexpr int NW = 8;          // waves per workgroup
constexpr int MERGE_LD = 132;  // floats per merge row of 128 dims

// the factor of the unnormalised outputs once the head's sink has joined
__device__ __forceinline__ float final_scale(const Args& A, int head, float m, float l) {
  if (!A.sink) return 1.f / l;
  const float s = A.sink[head] * LOG2E, t = fmaxf(m, s), a = exp2f(m - t);
  return a / (l * a + exp2f(s - t));
}

template <int NK, int NV, int MODS>
__device__ __forceinline__ void split_item(const Args& A, const int4 it, const int gk, char* smem) {
  constexpr int DK = 32 * NK, DV = 32 * NV;
  const int s = it.x, qb = it.y, nq = it.z & 0xff, part = (it.z >> 8) & 0xfff, nparts = it.z >> 20, pidx = it.w;
  const int cb = blockIdx.x, gv = gk / (A.G / A.GV), cols = nq * A.R;
  if (cb * 16 >= cols) return;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, g = lane >> 4, c = lane & 15;
  const int ctx = A.ctx_len[s], ql = A.q_len[s];
  const int pos0 = ctx - ql + qb;
  auto tok_of = [&](int col) { return min(col, cols - 1) / A.R; };
  auto head_of = [&](int col) {
    const int cc = min(col, cols - 1);
    return gk * A.R + cc - cc / A.R * A.R;
  };
  auto row_of = [&](int col) { return (size_t)(A.q_start[s] + qb + tok_of(col)) * A.H + head_of(col); };  // q row of a column
  const int cpos = pos0 + tok_of(cb * 16 + c);  // this column's position
  const int klo = first_key(A, cpos), cnb = blocks_of(A, cpos);
  const Mods<MODS> mods(A, head_of(cb * 16 + c));
  // the item's tiles of 16: pooled blocks, then token pages (the kept ones before the window's); this partition's share
  const int last = pos0 + nq - 1, nb = blocks_of(A, last), np = (nb + 15) >> 4;
  const int p_lo = first_key(A, pos0) >> 4, nkeep = kept_tiles(A, 16, p_lo), total = np + nkeep + ((last + 16) >> 4) - p_lo;
  auto page_of = [&](int t) { return t - np < nkeep ? t - np : p_lo + t - np - nkeep; };
  const int per = (total + nparts - 1) / nparts;
  const int t_begin = part * per, t_end = min(total, t_begin + per);
  const int* bt = A.block_table + (size_t)s * A.max_blocks;

  bf16x8 kf[NK], vf[NV];
  auto load = [&](int t) {
    if (t < np) {
      const size_t row = pooled_row(A, bt, min(16 * t + c, nb - 1), gk);
      const bf16 *k = (const bf16*)A.pk + row * DK + 8 * g, *v = (const bf16*)A.pv + row * DV + 8 * g;
#pragma unroll
      for (int m = 0; m < NK; ++m) kf[m] = *reinterpret_cast<const bf16x8*>(k + m * 32);
#pragma unroll
      for (int m = 0; m < NV; ++m) vf[m] = *reinterpret_cast<const bf16x8*>(v + m * 32);
    } else {
      const size_t page = bt[page_of(t)];
      const bf16 *k = (const bf16*)A.kp + (page * A.G + gk) * (DK * 16) + lane * 8;
      const bf16* v = (const bf16*)A.vp + (page * A.GV + gv) * (DV * 16) + lane * 8;
#pragma unroll
      for (int m = 0; m < NK; ++m) kf[m] = *reinterpret_cast<const bf16x8*>(k + m * 512);
#pragma unroll
      for (int m = 0; m < NV; ++m) vf[m] = *reinterpret_cast<const bf16x8*>(v + m * 512);
    }
  };
  // the wave's first tile is under way while the queries are staged
  if (t_begin + wid < t_end) load(t_begin + wid);
  char* sq = smem + NW * (DV * 32);
  for (int m = wid; m < NK; m += NW)
    *reinterpret_cast<bf16x8*>(sq + m * 1024 + lane * 16) =
        *reinterpret_cast<const bf16x8*>((const bf16*)A.q + row_of(cb * 16 + c) * DK + 32 * m + 8 * g);
  __syncthreads();
  f32x4 o[2 * NV];
#pragma unroll
  for (int n = 0; n < 2 * NV; ++n) o[n] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m_run = NEG_BIG, l_run = 0.f;
  char* my = smem + wid * (DV * 32);  // 16 keys x DV dims
  const int loff = lane * 16;         // this lane's 16 B of a k-step
  const int toff = ((c & 3) >> 1) * 256 + (4 * g + (c >> 2)) * 16 + (c & 1) * 8;

  for (int t = t_begin + wid; t < t_end; t += NW) {
    f32x4 s1[1] = {f32x4{0.f, 0.f, 0.f, 0.f}};
    f32x4& sc = s1[0];
#pragma unroll
    for (int m = 0; m < NK; ++m) {
      const bf16x8 qf = *reinterpret_cast<const bf16x8*>(sq + m * 1024 + loff);
      sc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[m], qf, sc, 0, 0, 0);
    }
#pragma unroll
    for (int m = 0; m < NV; ++m) *reinterpret_cast<bf16x8*>(my + m * 1024 + loff) = vf[m];
    if (t + NW < t_end) load(t + NW);
    mods.cap(s1);
    float tmax = NEG_BIG;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int e = 4 * g + r, key = 16 * page_of(t) + e;
      const bool ok = t < np ? 16 * t + e < cnb : (key <= cpos && (key >= klo || key < A.keep));
      if (MODS == BIAS && t >= np) sc[r] = fmaf(mods.slope, (float)(key - cpos), sc[r]);
      sc[r] = ok ? sc[r] * A.scale_log2 : NEG_BIG;
      tmax = fmaxf(tmax, sc[r]);
    }
    tmax = fmaxf(tmax, __shfl_xor(tmax, 16, 64));
    tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
    const float m_new = fmaxf(m_run, tmax);
    if (__any(m_new > m_run)) {
      const float alpha = exp2f(m_run - m_new);
      l_run *= alpha;
#pragma unroll
      for (int n = 0; n < 2 * NV; ++n) o[n] *= alpha;
      m_run = m_new;
    }
    bf16x4 pf;
    const float nm = m_run < 0.01f * NEG_BIG ? 0.f : m_run;  // (a column without a key yet: weights of 0)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float e = exp2f(sc[r] - nm);
      l_run += e;
      pf[r] = (bf16)e;
    }
    // the tile is private to the wave: its LDS operations complete in order
    const s16x4 pb = __builtin_bit_cast(s16x4, pf);
#pragma unroll
    for (int n = 0; n < 2 * NV; ++n) {
      const s16x4 v = __builtin_bit_cast(s16x4, tr_read(my + n * 512 + toff));
      o[n] = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(v, pb, o[n], 0, 0, 0);
    }
  }
  l_run += __shfl_xor(l_run, 16, 64);
  l_run += __shfl_xor(l_run, 32, 64);

  // merge the waves, 128 dims at a time
  float* mo = reinterpret_cast<float*>(smem);                           // [NW][16][MERGE_LD]
  float* mm = reinterpret_cast<float*>(smem + NW * 16 * MERGE_LD * 4);  // [NW][16]
  float* ml = mm + NW * 16;
  __syncthreads();
  if (g == 0) {
    mm[wid * 16 + c] = m_run;
    ml[wid * 16 + c] = l_run;
  }
  const int ccol = threadIdx.x >> 5, d4 = (threadIdx.x & 31) * 4;
  const bool cvalid = cb * 16 + ccol < cols;
  const size_t prow = (((size_t)gk * A.max_items + pidx) * A.NB + cb) * 16 + ccol;
  float wgt[NW], L = 0.f, mt = NEG_BIG;
#pragma unroll
  for (int b = 0; b < (NV + 3) / 4; ++b) {
    if (b) __syncthreads();
#pragma unroll
    for (int n = 0; n < 8; ++n)
      if (b * 8 + n < 2 * NV) *reinterpret_cast<f32x4*>(mo + (wid * 16 + c) * MERGE_LD + 16 * n + 4 * g) = o[b * 8 + n];
    __syncthreads();
    if (b == 0) {
#pragma unroll
      for (int w = 0; w < NW; ++w) mt = fmaxf(mt, mm[w * 16 + ccol]);
#pragma unroll
      for (int w = 0; w < NW; ++w) {
        wgt[w] = exp2f(mm[w * 16 + ccol] - mt);
        L += wgt[w] * ml[w * 16 + ccol];
      }
    }
    const int d0 = b * 128 + d4;
    if (d0 < DV) {
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int w = 0; w < NW; ++w)
        acc += wgt[w] * *reinterpret_cast<const f32x4*>(mo + (w * 16 + ccol) * MERGE_LD + d4);
      if (nparts > 1) {
        *reinterpret_cast<f32x4*>(A.part_o + prow * DV + d0) = acc;
      } else if (cvalid) {
        const int head = head_of(cb * 16 + ccol);
        const float f = final_scale(A, head, mt, L);
        float v[4] = {acc[0] * f, acc[1] * f, acc[2] * f, acc[3] * f};
        put_out<bf16>(A, (size_t)(A.q_start[s] + qb + tok_of(cb * 16 + ccol)), head, d0, v);
      }
    }
  }
  if (nparts > 1 && (threadIdx.x & 31) == 0) reinterpret_cast<float2*>(A.part_ml)[prow] = float2{mt, L};
}

// The partitions of an item, merged: a wave per (item, KV head, column), 4 dims per lane and step.
template <int NV>
__global__ __launch_bounds__(256) void merge_kernel(const Args A) {
  constexpr int DV = 32 * NV, NE = (DV + 255) / 256;
  const int lane = threadIdx.x & 63, gk = blockIdx.z;
  const int n = A.n_items[0];
  for (int item = blockIdx.y; item < n; item += gridDim.y) {
    const int4 it = A.items[item];
    const int nq = it.z & 0xff, nparts = it.z >> 20;
    if (nparts <= 1 || ((it.z >> 8) & 0xfff) != 0) continue;
    const int step = nq <= A.dec_tokens ? 1 : 8;  // slots of a partition
    for (int col = blockIdx.x * 4 + (threadIdx.x >> 6); col < nq * A.R; col += gridDim.x * 4) {
      auto slot = [&](int p) { return ((size_t)gk * A.max_items + it.w + p * step) * A.NB * 16 + col; };
      const float2* ml = reinterpret_cast<const float2*>(A.part_ml);
      float gm = NEG_BIG, L = 0.f;
      for (int p0 = 0; p0 < nparts; p0 += 64) gm = fmaxf(gm, p0 + lane < nparts ? ml[slot(p0 + lane)].x : NEG_BIG);
      gm = wave_max(gm);
      f32x4 a[NE];
#pragma unroll
      for (int e = 0; e < NE; ++e) a[e] = f32x4{0.f, 0.f, 0.f, 0.f};
      for (int p0 = 0; p0 < nparts; p0 += 64) {
        float w = 0.f;
        if (p0 + lane < nparts) {
          const float2 v = ml[slot(p0 + lane)];
          w = exp2f(v.x - gm);
          L += w * v.y;
        }
        const int np = min(64, nparts - p0);
#pragma unroll 8
        for (int p = 0; p < np; ++p) {
          const float wp = __shfl(w, p, 64);
#pragma unroll
          for (int e = 0; e < NE; ++e)
            a[e] += wp * *reinterpret_cast<const f32x4*>(A.part_o + slot(p0 + p) * DV + min(e * 256 + lane * 4, DV - 4));
        }
      }
      const int t = col / A.R, head = gk * A.R + col - t * A.R;
      const float f = final_scale(A, head, gm, wave_sum(L));
#pragma unroll
      for (int e = 0; e < NE; ++e) {
        const int d = e * 256 + lane * 4;
        float v[4] = {a[e][0] * f, a[e][1] * f, a[e][2] * f, a[e][3] * f};
        if (d < DV) put_out<bf16>(A, (size_t)(A.q_start[it.x] + it.y + t), head, d, v);
      }
    }
  }
}

template <int NK, int NV>
constexpr int tile_parts() { return NK + NV <= 8 ? 4 : 2; }  // 16-key parts of a tile

// Tiles run in the order of the items, all KV heads of one after the other (a head stays on its XCDs), but every second
// round of the 256 CUs from its end: the scheduler lists long items first, and a CU's workgroups then come to
// about the same number of keys.
__device__ __forceinline__ int tile_order(int i, int n, int G) {
  const int per = max(1, 256 / G), round = i / per;
  return round & 1 ? round * per + min(per, n - round * per) - 1 - (i - round * per) : i;
}

template <int NK, int NV, int MODS>
__device__ __forceinline__ void tile_item(const Args& A, const int4 it, const int gk, char* smem) {
  constexpr int DK = 32 * NK, DV = 32 * NV, KT = tile_parts<NK, NV>(), KEYS = 16 * KT;
  constexpr int PART = (NK + NV) * 1024, TILE = KT * PART;  // a 16-key part: K, then V
  const int s = it.x, qb = it.y, nq = it.z & 0xff, part = (it.z >> 8) & 0xfff, nparts = it.z >> 20;
  const int cols = nq * A.R, cw = blockIdx.x * (16 * NW), gv = gk / (A.G / A.GV);
  if (cw >= cols) return;
  const int lane = threadIdx.x & 63, wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, c = lane & 15;
  const int ctx = A.ctx_len[s], ql = A.q_len[s];
  const int pos0 = ctx - ql + qb;
  const int* bt = A.block_table + (size_t)s * A.max_blocks;
  const int ci = cw + wid * 16 + c, cc = min(ci, cols - 1), ct = cc / A.R;
  const int cpos = pos0 + ct, klo = first_key(A, cpos), cnb = blocks_of(A, cpos);
  const int row = (A.q_start[s] + qb + ct) * A.H + gk * A.R + cc - ct * A.R;  // of q
  const Mods<MODS> mods(A, gk * A.R + cc - ct * A.R);
  const int loff = lane * 16;
  bf16x8 qf[NK];
#pragma unroll
  for (int m = 0; m < NK; ++m) qf[m] = *reinterpret_cast<const bf16x8*>((const bf16*)A.q + (size_t)row * DK + 32 * m + 8 * g);
  // positions of the workgroup's columns -> its tiles: pooled blocks, then tokens (the kept before the window's)
  const int f = pos0 + cw / A.R, e = pos0 + min(cw + 16 * NW - 1, cols - 1) / A.R;
  const int nb = blocks_of(A, e), np = (nb + KEYS - 1) / KEYS;
  const int k_lo = first_key(A, f) / KEYS, nkeep = kept_tiles(A, KEYS, k_lo);
  int t_lo = 0, t_hi = np + nkeep + (e + KEYS) / KEYS - k_lo;
  auto tile_of = [&](int t) { return t - np < nkeep ? t - np : k_lo + t - np - nkeep; };
  if (nparts > 1) {  // this partition's tiles (possibly none)
    const int per = (t_hi + nparts - 1) / nparts;
    t_lo = part * per;
    t_hi = min(t_hi, t_lo + per);
  }
  const int nblk = (ctx + 15) >> 4;
  // this wave's columns: a tile whose keys all of them see needs no mask
  const int wf = pos0 + min(cw + wid * 16, cols - 1) / A.R;
  const int we = pos0 + min(cw + wid * 16 + 15, cols - 1) / A.R;
  const int full_lo = first_key(A, we), full_hi = wf, full_nb = blocks_of(A, wf);

  f32x4 o[2 * NV];
#pragma unroll
  for (int n = 0; n < 2 * NV; ++n) o[n] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m_run = NEG_BIG, l_run = 0.f;
  // direct loads, 1 KB per wave and instruction; a token page is copied linearly, pooled rows by lane. The
  // page ids of a wave's next chunks are read a tile ahead.
  constexpr int CHUNKS = KT * (NK + NV), PER = (CHUNKS + NW - 1) / NW;
  int pg[PER];
  auto pages = [&](int t) {
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int x = min((i * NW + wid) / (NK + NV), KT - 1);
      pg[i] = bt[min(max(KT * tile_of(t) + x, 0), nblk - 1)];
    }
  };
  auto issue = [&](int t, char* dst) {
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int ch = i * NW + wid;  // wave-uniform
      if (CHUNKS % NW == 0 || ch < CHUNKS) {
        const int x = ch / (NK + NV), m = ch - x * (NK + NV);
        const bf16* src;
        if (t < np) {
          const size_t r = pooled_row(A, bt, min(KEYS * t + 16 * x + c, nb - 1), gk);
          src = m < NK ? (const bf16*)A.pk + r * DK + 32 * m + 8 * g : (const bf16*)A.pv + r * DV + 32 * (m - NK) + 8 * g;
        } else {
          const size_t r = pg[i];
          src = (m < NK ? (const bf16*)A.kp + (r * A.G + gk) * (DK * 16) + m * 512
                        : (const bf16*)A.vp + (r * A.GV + gv) * (DV * 16) + (m - NK) * 512) + lane * 8;
        }
        __builtin_amdgcn_global_load_lds((glb_void*)src, (lds_void*)(dst + ch * 1024), 16, 0, 0);
      }
    }
  };
  const int toff = ((c & 3) >> 1) * 256 + (4 * g + (c >> 2)) * 16 + (c & 1) * 8;
  if (t_lo < t_hi) {
    pages(t_lo);
    issue(t_lo, smem);
    pages(t_lo + 1);
  }
  for (int t = t_lo; t < t_hi; ++t) {
    char* cur = smem + ((t - t_lo) & 1) * TILE;
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();  // tile t is whole, and nobody reads the other buffer any more
    if (t + 1 < t_hi) {
      issue(t + 1, smem + ((t + 1 - t_lo) & 1) * TILE);
      pages(t + 2);
    }
    f32x4 sc[KT];
#pragma unroll
    for (int k = 0; k < KT; ++k) sc[k] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int m = 0; m < NK; ++m)
#pragma unroll
      for (int k = 0; k < KT; ++k) {
        const bf16x8 kf = *reinterpret_cast<const bf16x8*>(cur + k * PART + m * 1024 + loff);
        sc[k] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[m], sc[k], 0, 0, 0);
      }
    const int key0 = KEYS * tile_of(t);  // wave-uniform
    float off = 0.f;  // of all this lane's scores
    mods.cap(sc);
    if (MODS == BIAS && t >= np) {
      off = mods.slope * (float)(key0 + 4 * g - cpos);
#pragma unroll
      for (int k = 0; k < KT; ++k)
#pragma unroll
        for (int r = 0; r < 4; ++r) sc[k][r] = fmaf(mods.slope, (float)(16 * k + r), sc[k][r]);
    }
    if (t < np ? KEYS * (t + 1) > full_nb
               : ((key0 < full_lo && key0 + KEYS > A.keep) || key0 + KEYS - 1 > full_hi)) {
#pragma unroll
      for (int k = 0; k < KT; ++k)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int x = 16 * k + 4 * g + r, key = key0 + x;
          if (t < np ? KEYS * t + x >= cnb : (key > cpos || (key < klo && key >= A.keep))) sc[k][r] = NEG_BIG;
        }
    }
    float tmax = NEG_BIG;
#pragma unroll
    for (int k = 0; k < KT; ++k)
#pragma unroll
      for (int r = 0; r < 4; ++r) tmax = fmaxf(tmax, sc[k][r]);
    if (MODS == BIAS) tmax += off;
    tmax = fmaxf(tmax, __shfl_xor(tmax, 16, 64));
    tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
    const float m_new = fmaxf(m_run, fmaxf(tmax * A.scale_log2, NEG_BIG));
    if (__any(m_new > m_run)) {
      const float alpha = exp2f(m_run - m_new);
      l_run *= alpha;
#pragma unroll
      for (int n = 0; n < 2 * NV; ++n) o[n] *= alpha;
      m_run = m_new;
    }
    // a column that has seen no key yet (its window starts in a later tile): every weight is 0
    float nm = m_run < 0.01f * NEG_BIG ? 0.f : -m_run;
    if (MODS == BIAS) nm = fmaf(off, A.scale_log2, nm);
    bf16x8 pf[KT / 2];
#pragma unroll
    for (int k = 0; k < KT; ++k)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float p = __builtin_amdgcn_exp2f(fmaf(sc[k][r], A.scale_log2, nm));
        l_run += p;
        pf[k / 2][4 * (k % 2) + r] = (bf16)p;
      }
#pragma unroll
    for (int k = 0; k < KT / 2; ++k)
#pragma unroll
      for (int n = 0; n < 2 * NV; ++n) {
        const char* vt = cur + 2 * k * PART + NK * 1024 + n * 512 + toff;
        const bf16x4 v0 = tr_read(vt), v1 = tr_read(vt + PART);
        bf16x8 v;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          v[j] = v0[j];
          v[4 + j] = v1[j];
        }
        o[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, pf[k], o[n], 0, 0, 0);
      }
  }
  l_run += __shfl_xor(l_run, 16, 64);
  l_run += __shfl_xor(l_run, 32, 64);
  if (ci >= cols) return;
  if (nparts > 1) {  // 8 slots hold the item's columns in a row
    const size_t pc = ((size_t)gk * A.max_items + it.w) * A.NB * 16 + ci;
    float* po = A.part_o + pc * DV + 4 * g;
#pragma unroll
    for (int n = 0; n < 2 * NV; ++n) *reinterpret_cast<f32x4*>(po + 16 * n) = o[n];
    if (g == 0) reinterpret_cast<float2*>(A.part_ml)[pc] = float2{m_run, l_run};
    return;
  }
  const int tok = row / A.H, head = row - tok * A.H;
  const float fs = final_scale(A, head, m_run, l_run);
#pragma unroll
  for (int n = 0; n < 2 * NV; ++n) {
    float v[4] = {o[n][0] * fs, o[n][1] * fs, o[n][2] * fs, o[n][3] * fs};
    put_out<bf16>(A, (size_t)tok, head, 16 * n + 4 * g, v);
  }
}

template <int NK, int NV>
constexpr int lds_bytes() {
  return std::max({2 * tile_parts<NK, NV>() * 1024 * (NK + NV), NW * 32 * 32 * NV + 1024 * NK, NW * 16 * MERGE_LD * 4 + 2 * NW * 16 * 4});
}

// The two paths want different registers: tiles four waves a SIMD, split items all they can hold. Small steps
// run both in one launch, larger ones each in its own.
enum { TILES = 1, SPLITS = 2 };

template <int NK, int NV, int PATHS, int MODS>
__global__ __launch_bounds__(64 * NW, (PATHS == TILES && NK + NV <= 8) || NK + NV <= 6 ? 4 : 2) void mfma_kernel(const Args A) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int n = A.n_items[0];
  // two passes over the workgroup's items, so that neither path's registers carry the other's
  if constexpr ((PATHS & TILES) != 0)
    for (int w = blockIdx.y; w < n * A.G; w += gridDim.y) {
      const int4 it = A.items[tile_order(w / A.G, n, A.G)];
      if ((it.z & 0xff) <= A.dec_tokens) continue;
      tile_item<NK, NV, MODS>(A, it, w % A.G, smem);
      __syncthreads();
    }
  if constexpr ((PATHS & SPLITS) != 0)
    for (int w = blockIdx.y; w < n * A.G; w += gridDim.y) {
      const int4 it = A.items[w / A.G];
      if ((it.z & 0xff) > A.dec_tokens) continue;
      split_item<NK, NV, MODS>(A, it, w % A.G, smem);
      __syncthreads();
    }
}

}  // namespace wa
}  // namespace pa

// (key width, value width) in 32s with MFMA kernels, smallest first
#define PA_WA_DIMS(X) \
  X(1, 1) X(1, 2) X(2, 1) X(2, 2) X(2, 4) X(3, 3) X(4, 2) X(4, 4) X(4, 8) X(6, 4) X(6, 6) X(8, 8)

// The padded widths for key size k and value size v: the first built pair that holds both, else whole
// 32s (the simple kernel then runs).
extern "C" void pa_window_pad(int k, int v, int* dk, int* dv) {
  const int a = (k + 31) / 32, b = (v + 31) / 32;
#define PA_X(K, V)         \
  if (a <= K && b <= V) {  \
    *dk = 32 * K;          \
    *dv = 32 * V;          \
    return;                \
  }
  PA_WA_DIMS(PA_X)
#undef PA_X
  *dk = 32 * a;
  *dv = 32 * b;
}

extern "C" int pa_window_attention(int fp32, void* out, int out_f32, int ldo, float* part_o, float* part_ml, const void* q,
                                   const void* kp, const void* vp, const void* pk, const void* pv, const int* items,
                                   const int* n_items, int max_items, const int* q_start, const int* q_len,
                                   const int* ctx_len, const int* block_table, int max_blocks, int T, int H, int G, int GV,
                                   int DK, int DV, int dec_tokens, int tile_tokens, int window, int pool, int npb, int keep,
                                   int chunk, int max_slots, float scale, const float* slopes, float cap, const float* sink,
                                   const void* gate, int ldg, float gain, int simple, hipStream_t st) {
  if (max_items <= 0) return 0;
  if (DK % 32 || DV % 32 || H <= 0 || G <= 0 || GV <= 0 || H % G || G % GV || dec_tokens <= 0 || tile_tokens <= 0) return -1;
  if (scale <= 0.f || keep < 0 || (keep > 0 && window <= 0) || (chunk > 0 && window > 0) || ldo % 4 || (gate && ldg % 4) ||
      (pool > 0 && (keep > 0 || chunk > 0 || G != GV))) return -1;
  const int R = H / G, NB = (dec_tokens * R + 15) / 16;
  pa::wa::Args A{out, part_o, part_ml, q, kp, vp, pk, pv, (const int4*)items, n_items, q_start, q_len, ctx_len,
                 block_table, max_blocks, max_slots, H, G, R, NB, DK, DV, dec_tokens, window, pool, npb,
                 scale * pa::wa::LOG2E, sink, slopes, gate, scale, cap, gain, GV, keep, chunk, ldo, ldg, out_f32};
  if (!fp32 && !simple) {
    const int cw = 16 * pa::wa::NW, gt = (tile_tokens * R + cw - 1) / cw, gx = NB > gt ? NB : gt;
    const int gi = std::min(max_items, std::max(256, 2048 / G)), gy = gi * G;  // (workgroups loop over the rest)
#define PA_KERNELS(K, V, M)                                                                                   \
  do {                                                                                                        \
    constexpr int lds = lds_bytes<K, V>();                                                                    \
    static bool attr = false;                                                                                 \
    if (!attr) {                                                                                              \
      for (const void* f : {(const void*)mfma_kernel<K, V, TILES, M>, (const void*)mfma_kernel<K, V, SPLITS, M>, \
                            (const void*)mfma_kernel<K, V, TILES | SPLITS, M>})                               \
        (void)hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, lds);                        \
      attr = true;                                                                                            \
    }                                                                                                         \
    const dim3 wg(64 * NW);                                                                                   \
    if (T <= 64) {                                                                                            \
      hipLaunchKernelGGL((mfma_kernel<K, V, TILES | SPLITS, M>), dim3(gx, gy), wg, lds, st, A);            \
    } else {                                                                                                  \
      hipLaunchKernelGGL((mfma_kernel<K, V, TILES, M>), dim3(gt, gy), wg, lds, st, A);                     \
      hipLaunchKernelGGL((mfma_kernel<K, V, SPLITS, M>), dim3(NB, gy), wg, lds, st, A);                    \
    }                                                                                                         \
  } while (0)
#define PA_X(K, V)                                                                                            \
  if (DK == 32 * K && DV == 32 * V) {                                                                         \
    using namespace pa::wa;                                                                                   \
    if (slopes) PA_KERNELS(K, V, BIAS);                                                                       \
    else if (cap > 0.f) PA_KERNELS(K, V, CAP);                                                                \
    else PA_KERNELS(K, V, NO_MODS);                                                                           \
    hipLaunchKernelGGL((pa::wa::merge_kernel<V>), dim3(T <= 64 || T > 1024 ? 8 : 16, std::min(gi, 64), G), dim3(256), 0, st, A);        \
    return (int)hipGetLastError();                                                                            \
  }
    PA_WA_DIMS(PA_X)
#undef PA_X
#undef PA_KERNELS
  }
  if (DV > 2048 || DK > 8192) return -2;
  const dim3 grid(H, max_items < 4096 ? max_items : 4096);
  const int lds = (DK + 256 + 4) * 4;
  if (fp32) hipLaunchKernelGGL((pa::wa::simple_kernel<float>), grid, dim3(256), lds, st, A);
  else hipLaunchKernelGGL((pa::wa::simple_kernel<pa::bf16>), grid, dim3(256), lds, st, A);
  return (int)hipGetLastError();
}
