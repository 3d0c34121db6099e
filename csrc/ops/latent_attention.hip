// Paged latent attention (queries absorbed into the latent space), for prefill chunks, decode
// rows and mixed batches in one launch.
//
// The cache holds one row per token for all heads: [latent c (Rp) | rotated key part (rp)],
// D = Rp + rp (rp 0: a latent without positions), pages of 16 tokens, fragment-major [D/8][16][8] (latent_cache.hip). With
//   q~_h = [W_uk,h^T q_h | rot(q_h)]          (absorbed before the launch)
//   score_h(i, j) = q~_h(i) . row(j) * scale,  o~_h(i) = sum_j softmax_j score * c(j)
// every head reads the same rows: keys are the whole row, values its first Rp dims, and the
// W_uv up-projection of o~ follows the launch. The MFMA columns are (token, head) pairs,
// consecutive rows of q~ [T, H, D], so any head count fills them.
//
//   S^T[keys x cols] = rows . Q^T      A = key rows (one 1-KB run of a page per k-step), B = Q^T
//   O^T[dims x cols] += c^T . P^T      A = c^T by LDS transpose reads (ds_read_b64_tr_b16) of the
//                                      SAME tile, B = P^T = the S^T accumulator's own registers
// so the rows are read from HBM once and stored once; no transposed copy exists anywhere.
//
// A window of W keys (0: none) limits position i to keys i - W + 1 .. i: tiles wholly outside an
// item's range are never read.
//
// Items come from the scheduler like paged_attention's (seq, q_begin, nq | part<<8 | nparts<<20,
// partial slot):
//   nq <= dec_tokens: split over keys. The 8 waves take every 8th page with a private LDS tile and
//                     merge; nparts > 1 divides the item's own (windowed) key range evenly, the
//                     partials go to memory and merge_kernel, a second launch, combines them: at
//                     16 x Rp floats a partition, one last arriver would read for longer than all
//                     partitions compute, while the launch spreads the columns over the chip.
//   otherwise:        128 columns per workgroup, 16 per wave; all waves share double-buffered 32-key
//                     tiles that arrive by direct global -> LDS loads. A step with few such items
//                     has them cut into partitions of their keys too (8 slots each).
#include "common.h"

#include <algorithm>

namespace pa {
namespace la {

constexpr float NEG_BIG = -1.0e30f;
typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) bf16x4 lds_bf16x4;
typedef __attribute__((address_space(3))) void lds_void;
typedef const __attribute__((address_space(1))) void glb_void;

struct Args {
  void* out;             // [T, H, Rp]
  float* part_o;         // [slots, NB, 16, Rp]
  float* part_ml;        // [slots, NB, 16, 2]
  const void* q;         // [T, H, D]
  const void* pages;
  const int4* items;
  const int* n_items;
  const int *q_start, *q_len, *ctx_len, *block_table;
  int max_blocks, H, NB, Rp, D, dec_tokens, window;
  float scale_log2;
};

// ---------------------------------------------------------------------------
// Any sizes, bf16 or fp32: one workgroup per (token of an item, head). The exact path.
template <typename T>
__global__ __launch_bounds__(256) void simple_kernel(const Args A) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float* sq = sm;           // D
  float* sp = sm + A.D;     // 256
  float* red = sp + 256;    // 4
  const int h = blockIdx.x, n = A.n_items[0];
  for (int item = blockIdx.y; item < n; item += gridDim.y) {
    const int4 it = A.items[item];
    const int s = it.x, nq = it.z & 0xff, part = (it.z >> 8) & 0xfff;
    if (part > 0) continue;  // partition 0 takes the whole range
    const int ctx = A.ctx_len[s], ql = A.q_len[s];
    const int* bt = A.block_table + (size_t)s * A.max_blocks;
    for (int i = 0; i < nq; ++i) {
      const int tok = it.y + i, pos = ctx - ql + tok;
      const int lo = A.window > 0 ? max(0, pos - A.window + 1) : 0;
      const size_t row = (size_t)(A.q_start[s] + tok) * A.H + h;
      __syncthreads();
      for (int d = threadIdx.x; d < A.D; d += 256) sq[d] = (float)((const T*)A.q)[row * A.D + d];
      __syncthreads();
      float m = NEG_BIG, l = 0.f, o[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
      for (int k0 = lo; k0 <= pos; k0 += 256) {
        const int key = k0 + threadIdx.x;
        float sc = NEG_BIG;
        if (key <= pos) {
          const T* kr = (const T*)A.pages + (size_t)bt[key >> 4] * A.D * 16 + (key & 15) * 8;
          float a = 0.f;
          for (int d = 0; d < A.D; d += 8)
#pragma unroll
            for (int j = 0; j < 8; ++j) a += sq[d + j] * (float)kr[(size_t)d * 16 + j];
          sc = a * A.scale_log2;
        }
        const float wm = wave_max(sc);
        if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = wm;
        __syncthreads();
        const float mn = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
        const float alpha = exp2f(m - mn), p = key <= pos ? exp2f(sc - mn) : 0.f;
        m = mn;
        sp[threadIdx.x] = p;
        __syncthreads();
        l = l * alpha + block_sum<4>(p, red);
        const int nk = min(256, pos + 1 - k0);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const int d = threadIdx.x + 256 * e;
          if (d >= A.Rp) break;
          float a = o[e] * alpha;
          for (int k = 0; k < nk; ++k) {
            const int kk = k0 + k;
            a += sp[k] * (float)((const T*)A.pages)[(size_t)bt[kk >> 4] * A.D * 16 + (size_t)(d >> 3) * 128 +
                                                    (kk & 15) * 8 + (d & 7)];
          }
          o[e] = a;
        }
        __syncthreads();
      }
      const float inv = 1.f / l;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int d = threadIdx.x + 256 * e;
        if (d < A.Rp) ((T*)A.out)[row * A.Rp + d] = (T)(o[e] * inv);
      }
    }
  }
}

// ---------------------------------------------------------------------------
// c^T operand: lanes 16g + i of the result hold dim i of keys 4g .. 4g + 3; each lane names the
// 8 bytes (key 4g + i/4, dims 4 (i%4) .. + 3) of the 4 x 16 block its group transposes
__device__ __forceinline__ bf16x4 tr_read(const char* p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds_bf16x4*)p);
}

constexpr int NW = 8;          // waves per workgroup: two a SIMD, one's softmax under the other's MFMAs
constexpr int MERGE_LD = 132;  // floats per merge row of 128 dims

template <int RT, int PT>
__device__ __forceinline__ void split_item(const Args& A, const int4 it, char* smem) {
  constexpr int NK = RT + PT, D = 32 * NK, RP = 32 * RT;
  const int s = it.x, qb = it.y, nq = it.z & 0xff, part = (it.z >> 8) & 0xfff, nparts = it.z >> 20, pidx = it.w;
  const int cb = blockIdx.x, cols = nq * A.H;
  if (cb * 16 >= cols) return;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, g = lane >> 4, c = lane & 15;
  const int ctx = A.ctx_len[s], ql = A.q_len[s];
  const int pos0 = ctx - ql + qb;
  const int ci = cb * 16 + c;
  const int cpos = pos0 + min(ci, cols - 1) / A.H;  // this column's position
  const int klo = A.window > 0 ? max(0, cpos - A.window + 1) : 0;
  const size_t row0 = (size_t)(A.q_start[s] + qb) * A.H + cb * 16;  // q~ row of column 0
  const size_t row = row0 + min(c, cols - 1 - cb * 16);
  // the item's pages, and this partition's share
  const int p_lo = (A.window > 0 ? max(0, pos0 - A.window + 1) : 0) >> 4, p_hi = (pos0 + nq + 15) >> 4;
  const int per = (p_hi - p_lo + nparts - 1) / nparts;
  const int p_begin = p_lo + part * per, p_end = min(p_hi, p_begin + per);
  const int* bt = A.block_table + (size_t)s * A.max_blocks;

  constexpr bool AHEAD = RT < 16;
  bf16x8 kf[NK];
  auto load = [&](int p, bf16x8 (&k)[NK]) {
    const bf16* b = (const bf16*)A.pages + (size_t)bt[p] * (D * 16) + (g * 16 + c) * 8;
#pragma unroll
    for (int m = 0; m < NK; ++m) k[m] = *reinterpret_cast<const bf16x8*>(b + m * 512);
  };
  // the wave's first page is under way while the queries are staged
  if (AHEAD && p_begin + wid < p_end) load(p_begin + wid, kf);
  // all waves share the 16 columns: their Q^T operands (1 KB per k-step) live in LDS
  char* sq = smem + NW * (RP * 32);
  for (int m = wid; m < NK; m += NW)
    *reinterpret_cast<bf16x8*>(sq + m * 1024 + (g * 16 + c) * 16) =
        *reinterpret_cast<const bf16x8*>((const bf16*)A.q + row * D + 32 * m + 8 * g);
  __syncthreads();
  f32x4 o[2 * RT];
#pragma unroll
  for (int n = 0; n < 2 * RT; ++n) o[n] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m_run = NEG_BIG, l_run = 0.f;
  char* my = smem + wid * (RP * 32);  // 16 keys x RP dims
  const int loff = (g * 16 + c) * 16;  // this lane's 16 B of a k-step
  const int toff = ((c & 3) >> 1) * 256 + (4 * g + (c >> 2)) * 16 + (c & 1) * 8;

  // the widest latents load a later page when they need it: it does not fit the registers beside the
  // outputs' update, and the SIMD's other wave computes meanwhile
  for (int p = p_begin + wid; p < p_end; p += NW) {
    if (!AHEAD) load(p, kf);
    f32x4 sc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int m = 0; m < NK; ++m) {
      const bf16x8 qf = *reinterpret_cast<const bf16x8*>(sq + m * 1024 + loff);
      sc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[m], qf, sc, 0, 0, 0);
      if (m < RT) *reinterpret_cast<bf16x8*>(my + m * 1024 + loff) = kf[m];
    }
    if (AHEAD && p + NW < p_end) load(p + NW, kf);
    float tmax = NEG_BIG;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int key = 16 * p + 4 * g + r;
      sc[r] = (key <= cpos && key >= klo) ? sc[r] * A.scale_log2 : NEG_BIG;
      tmax = fmaxf(tmax, sc[r]);
    }
    tmax = fmaxf(tmax, __shfl_xor(tmax, 16, 64));
    tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
    const float m_new = fmaxf(m_run, tmax);
    if (__any(m_new > m_run)) {
      const float alpha = exp2f(m_run - m_new);
      l_run *= alpha;
#pragma unroll
      for (int n = 0; n < 2 * RT; ++n) o[n] *= alpha;
      m_run = m_new;
    }
    bf16x4 pf;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float e = exp2f(sc[r] - m_run);
      l_run += e;
      pf[r] = (bf16)e;
    }
    // the tile is private to the wave: its LDS operations complete in order
    const s16x4 pb = __builtin_bit_cast(s16x4, pf);
#pragma unroll
    for (int n = 0; n < 2 * RT; ++n) {
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
  float wgt[NW], L = 0.f, mt = NEG_BIG;
#pragma unroll
  for (int nb = 0; nb < (RT + 3) / 4; ++nb) {
    if (nb) __syncthreads();
#pragma unroll
    for (int n = 0; n < 8; ++n)
      if (nb * 8 + n < 2 * RT) *reinterpret_cast<f32x4*>(mo + (wid * 16 + c) * MERGE_LD + 16 * n + 4 * g) = o[nb * 8 + n];
    __syncthreads();
    if (nb == 0) {
#pragma unroll
      for (int w = 0; w < NW; ++w) mt = fmaxf(mt, mm[w * 16 + ccol]);
#pragma unroll
      for (int w = 0; w < NW; ++w) {
        wgt[w] = exp2f(mm[w * 16 + ccol] - mt);
        L += wgt[w] * ml[w * 16 + ccol];
      }
    }
    const int d0 = nb * 128 + d4;
    if (d0 < RP) {
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int w = 0; w < NW; ++w)
        acc += wgt[w] * *reinterpret_cast<const f32x4*>(mo + (w * 16 + ccol) * MERGE_LD + d4);
      if (nparts > 1) {
        *reinterpret_cast<f32x4*>(A.part_o + (((size_t)pidx * A.NB + cb) * 16 + ccol) * RP + d0) = acc;
      } else if (cvalid) {
        const float inv = 1.f / L;
        bf16x4 v;
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] = (bf16)(acc[j] * inv);
        *reinterpret_cast<bf16x4*>((bf16*)A.out + (row0 + ccol) * RP + d0) = v;
      }
    }
  }
  if (nparts > 1 && (threadIdx.x & 31) == 0)
    reinterpret_cast<float2*>(A.part_ml)[((size_t)pidx * A.NB + cb) * 16 + ccol] = float2{mt, L};
}

// The partitions of an item, merged: a wave per (item, column), 8 dims per lane and step.
template <int RT>
__global__ __launch_bounds__(256) void merge_kernel(const Args A) {
  constexpr int RP = 32 * RT;
  const int lane = threadIdx.x & 63;
  const int n = A.n_items[0];
  for (int item = blockIdx.y; item < n; item += gridDim.y) {
    const int4 it = A.items[item];
    const int nq = it.z & 0xff, nparts = it.z >> 20;
    if (nparts <= 1 || ((it.z >> 8) & 0xfff) != 0) continue;
    const int step = nq <= A.dec_tokens ? 1 : 8;  // slots of a partition
    for (int col = blockIdx.x * 4 + (threadIdx.x >> 6); col < nq * A.H; col += gridDim.x * 4) {
      auto slot = [&](int p) { return (size_t)(it.w + p * step) * A.NB * 16 + col; };
      const float2* ml = reinterpret_cast<const float2*>(A.part_ml);
      // lane p holds partition p's weight (64 at a time): the loads of a round are independent
      float gm = NEG_BIG, L = 0.f;
      for (int p0 = 0; p0 < nparts; p0 += 64) gm = fmaxf(gm, p0 + lane < nparts ? ml[slot(p0 + lane)].x : NEG_BIG);
      gm = wave_max(gm);
      float a[(RP + 511) / 512][8];
#pragma unroll
      for (int e = 0; e < (RP + 511) / 512; ++e)
#pragma unroll
        for (int j = 0; j < 8; ++j) a[e][j] = 0.f;
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
          for (int e = 0; e < (RP + 511) / 512; ++e) {
            const int d = min(e * 512 + lane * 8, RP - 8);
            const f32x4* s = reinterpret_cast<const f32x4*>(A.part_o + slot(p0 + p) * RP + d);
            const f32x4 x = s[0], y = s[1];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
              a[e][j] += wp * x[j];
              a[e][4 + j] += wp * y[j];
            }
          }
        }
      }
      L = wave_sum(L);
      const float inv = 1.f / L;
      bf16* o = (bf16*)A.out + ((size_t)(A.q_start[it.x] + it.y) * A.H + col) * RP;
#pragma unroll
      for (int e = 0; e < (RP + 511) / 512; ++e) {
        const int d = e * 512 + lane * 8;
        if (d < RP) {
          bf16x8 v;
#pragma unroll
          for (int j = 0; j < 8; ++j) v[j] = (bf16)(a[e][j] * inv);
          *reinterpret_cast<bf16x8*>(o + d) = v;
        }
      }
    }
  }
}

template <int RT, int PT, int CT>
__device__ __forceinline__ void tile_item(const Args& A, const int4 it, char* smem) {
  constexpr int NK = RT + PT, D = 32 * NK, RP = 32 * RT, TILE = 32 * D * 2;
  const int s = it.x, qb = it.y, nq = it.z & 0xff, part = (it.z >> 8) & 0xfff, nparts = it.z >> 20;
  const int cols = nq * A.H, cw = blockIdx.x * (16 * NW * CT);
  if (cw >= cols) return;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, g = lane >> 4, c = lane & 15;
  const int ctx = A.ctx_len[s], ql = A.q_len[s];
  const int pos0 = ctx - ql + qb;
  const size_t row0 = (size_t)(A.q_start[s] + qb) * A.H;
  const int* bt = A.block_table + (size_t)s * A.max_blocks;
  int ci[CT], cpos[CT], klo[CT];
  // the widest rows keep their rotated part's queries in LDS (lane-private, above the key tiles)
  constexpr int NQ = NK > 17 ? RT : NK;
  const int loff = (g * 16 + c) * 16;
  char* qs = smem + 2 * TILE + wid * (CT * (NK - NQ) * 1024) + loff;
  bf16x8 qf[CT][NQ];
#pragma unroll
  for (int t = 0; t < CT; ++t) {
    ci[t] = cw + (wid * CT + t) * 16 + c;
    const int cc = min(ci[t], cols - 1);
    cpos[t] = pos0 + cc / A.H;
    klo[t] = A.window > 0 ? max(0, cpos[t] - A.window + 1) : 0;
#pragma unroll
    for (int m = 0; m < NK; ++m) {
      const bf16x8 v = *reinterpret_cast<const bf16x8*>((const bf16*)A.q + (row0 + cc) * D + 32 * m + 8 * g);
      if (m < NQ) qf[t][m] = v;
      else *reinterpret_cast<bf16x8*>(qs + (t * (NK - NQ) + m - NQ) * 1024) = v;
    }
  }
  // positions of the workgroup's columns -> its key tiles
  const int f = pos0 + cw / A.H, e = pos0 + min(cw + 16 * NW * CT - 1, cols - 1) / A.H;
  int t_lo = (A.window > 0 ? max(0, f - A.window + 1) : 0) >> 5, t_hi = (e + 32) >> 5;
  if (nparts > 1) {  // this partition's tiles (possibly none)
    const int per = (t_hi - t_lo + nparts - 1) / nparts;
    t_lo += part * per;
    t_hi = min(t_hi, t_lo + per);
  }
  const int nblk = (ctx + 15) >> 4;
  // this wave's columns: keys below all of their windows' starts / above all positions are masked
  // (t needs no mask when every column sees all its 32 keys)
  const int wf = pos0 + min(cw + wid * CT * 16, cols - 1) / A.H;
  const int we = pos0 + min(cw + wid * CT * 16 + 16 * CT - 1, cols - 1) / A.H;
  const int full_lo = A.window > 0 ? we - A.window + 1 : 0, full_hi = wf;

  f32x4 o[CT][2 * RT];
#pragma unroll
  for (int t = 0; t < CT; ++t)
#pragma unroll
    for (int n = 0; n < 2 * RT; ++n) o[t][n] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m_run[CT], l_run[CT];
#pragma unroll
  for (int t = 0; t < CT; ++t) {
    m_run[t] = NEG_BIG;
    l_run[t] = 0.f;
  }
  // direct loads: the tile is two whole pages, copied linearly, 1 KB per wave and instruction
  auto issue = [&](int t, char* dst) {
    const bf16* src0 = (const bf16*)A.pages + (size_t)bt[min(2 * t, nblk - 1)] * (D * 16) + lane * 8;
    const bf16* src1 = (const bf16*)A.pages + (size_t)bt[min(2 * t + 1, nblk - 1)] * (D * 16) + lane * 8;
#pragma unroll
    for (int i = 0; i < (2 * NK + NW - 1) / NW; ++i) {
      const int ch = i * NW + wid;  // wave-uniform
      if (2 * NK % NW == 0 || ch < 2 * NK)
        __builtin_amdgcn_global_load_lds((glb_void*)((ch < NK ? src0 : src1 - NK * 512) + ch * 512),
                                         (lds_void*)(dst + ch * 1024), 16, 0, 0);
    }
  };
  const int toff = ((c & 3) >> 1) * 256 + (4 * g + (c >> 2)) * 16 + (c & 1) * 8;
  if (t_lo < t_hi) issue(t_lo, smem);
  for (int t = t_lo; t < t_hi; ++t) {
    char* cur = smem + ((t - t_lo) & 1) * TILE;
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();  // tile t is whole, and nobody reads the other buffer any more
    if (t + 1 < t_hi) issue(t + 1, smem + ((t + 1 - t_lo) & 1) * TILE);
    f32x4 sc[CT][2];
#pragma unroll
    for (int x = 0; x < CT; ++x)
#pragma unroll
      for (int k = 0; k < 2; ++k) sc[x][k] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int m = 0; m < NK; ++m)
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const bf16x8 kf = *reinterpret_cast<const bf16x8*>(cur + k * (D * 32) + m * 1024 + loff);
#pragma unroll
        for (int x = 0; x < CT; ++x) {
          const bf16x8 q = m < NQ ? qf[x][m < NQ ? m : 0]
                                  : *reinterpret_cast<const bf16x8*>(qs + (x * (NK - NQ) + m - NQ) * 1024);
          sc[x][k] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, q, sc[x][k], 0, 0, 0);
        }
      }
    const bool mask = 32 * t < full_lo || 32 * t + 31 > full_hi;  // wave-uniform
    bf16x8 pf[CT];
#pragma unroll
    for (int x = 0; x < CT; ++x) {
      if (mask) {
#pragma unroll
        for (int k = 0; k < 2; ++k)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int key = 32 * t + 16 * k + 4 * g + r;
            if (key > cpos[x] || key < klo[x]) sc[x][k][r] = NEG_BIG;
          }
      }
      float tmax = NEG_BIG;
#pragma unroll
      for (int k = 0; k < 2; ++k)
#pragma unroll
        for (int r = 0; r < 4; ++r) tmax = fmaxf(tmax, sc[x][k][r]);
      tmax = fmaxf(tmax, __shfl_xor(tmax, 16, 64));
      tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
      const float m_new = fmaxf(m_run[x], fmaxf(tmax * A.scale_log2, NEG_BIG));
      if (__any(m_new > m_run[x])) {
        const float alpha = exp2f(m_run[x] - m_new);
        l_run[x] *= alpha;
#pragma unroll
        for (int n = 0; n < 2 * RT; ++n) o[x][n] *= alpha;
        m_run[x] = m_new;
      }
      // a column that has seen no key yet (its window starts in a later tile): every weight is 0
      const float nm = m_run[x] < 0.01f * NEG_BIG ? 0.f : -m_run[x];
#pragma unroll
      for (int k = 0; k < 2; ++k)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float p = __builtin_amdgcn_exp2f(fmaf(sc[x][k][r], A.scale_log2, nm));
          l_run[x] += p;
          pf[x][4 * k + r] = (bf16)p;
        }
    }
#pragma unroll
    for (int n = 0; n < 2 * RT; ++n) {
      const bf16x4 v0 = tr_read(cur + n * 512 + toff), v1 = tr_read(cur + D * 32 + n * 512 + toff);
      bf16x8 v;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        v[j] = v0[j];
        v[4 + j] = v1[j];
      }
#pragma unroll
      for (int x = 0; x < CT; ++x) o[x][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, pf[x], o[x][n], 0, 0, 0);
    }
  }
#pragma unroll
  for (int x = 0; x < CT; ++x) {
    float l = l_run[x];
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (ci[x] >= cols) continue;
    if (nparts > 1) {  // 8 slots hold the item's columns in a row
      const size_t pc = (size_t)it.w * A.NB * 16 + ci[x];
      float* po = A.part_o + pc * RP + 4 * g;
#pragma unroll
      for (int n = 0; n < 2 * RT; ++n) *reinterpret_cast<f32x4*>(po + 16 * n) = o[x][n];
      if (g == 0) reinterpret_cast<float2*>(A.part_ml)[pc] = float2{m_run[x], l};
      continue;
    }
    const float inv = 1.f / l;
    bf16* orow = (bf16*)A.out + (row0 + ci[x]) * RP + 4 * g;
#pragma unroll
    for (int n = 0; n < 2 * RT; ++n) {
      bf16x4 v;
#pragma unroll
      for (int r = 0; r < 4; ++r) v[r] = (bf16)(o[x][n][r] * inv);
      *reinterpret_cast<bf16x4*>(orow + 16 * n) = v;
    }
  }
}

template <int RT, int PT>
constexpr int lds_bytes() {
  return std::max({2 * 32 * 32 * (RT + PT) * 2 + (RT + PT > 17 ? NW * PT * 1024 : 0), NW * 32 * 32 * RT + 1024 * (RT + PT),
                   NW * 16 * MERGE_LD * 4 + 2 * NW * 16 * 4});
}

template <int RT, int PT, int CT>
__global__ __launch_bounds__(64 * NW, 2) void mfma_kernel(const Args A) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int n = A.n_items[0];
  // two passes over the workgroup's items, so that neither path's registers carry the other's
  for (int item = blockIdx.y; item < n; item += gridDim.y) {
    const int4 it = A.items[item];
    if ((it.z & 0xff) <= A.dec_tokens) continue;
    tile_item<RT, PT, CT>(A, it, smem);
    __syncthreads();
  }
  for (int item = blockIdx.y; item < n; item += gridDim.y) {
    const int4 it = A.items[item];
    if ((it.z & 0xff) > A.dec_tokens) continue;
    split_item<RT, PT>(A, it, smem);
    __syncthreads();
  }
}

}  // namespace la
}  // namespace pa

#define PA_LA_RT(X) X(1) X(2) X(3) X(4) X(6) X(8) X(12) X(16)

// The padded latent width the MFMA kernels use for R (the smallest built size that holds it), or
// R rounded to 32 when none does (the simple kernel then runs); likewise the rotated part.
extern "C" int pa_latent_pad(int R) {
  const int need = (R + 31) / 32;
#define PA_X(N) if (need <= N) return N * 32;
  PA_LA_RT(PA_X)
#undef PA_X
  return need * 32;
}

extern "C" int pa_latent_attention(int fp32, void* out, float* part_o, float* part_ml, const void* q, const void* pages, const int* items, const int* n_items, int max_items,
                                   const int* q_start, const int* q_len, const int* ctx_len, const int* block_table,
                                   int max_blocks, int H, int Rp, int rp, int dec_tokens, int tile_tokens, int window,
                                   float scale_log2, int simple, hipStream_t st) {
  if (max_items <= 0) return 0;
  const int D = Rp + rp, NB = (dec_tokens * H + 15) / 16;
  if (Rp % 32 || rp % 32 || H <= 0 || dec_tokens <= 0 || tile_tokens <= 0) return -1;
  pa::la::Args A{out, part_o, part_ml, q, pages, (const int4*)items, n_items, q_start, q_len, ctx_len,
                 block_table, max_blocks, H, NB, Rp, D, dec_tokens, window, scale_log2};
  const int RT = Rp / 32, PT = rp / 32;
  if (!fp32 && !simple && PT <= 2) {
#define PA_LA(R, P)                                                                                           \
  do {                                                                                                        \
    constexpr int CT = 1;                                                                                     \
    constexpr int lds = pa::la::lds_bytes<R, P>();                                                            \
    static bool attr = false;                                                                                 \
    if (!attr) {                                                                                              \
      (void)hipFuncSetAttribute((const void*)pa::la::mfma_kernel<R, P, CT>,                                   \
                                hipFuncAttributeMaxDynamicSharedMemorySize, lds);                             \
      attr = true;                                                                                            \
    }                                                                                                         \
    const int cw = 16 * pa::la::NW * CT, gt = (tile_tokens * H + cw - 1) / cw, gx = NB > gt ? NB : gt;                       \
    /* items are strided over the grid: at least one workgroup per CU */                                      \
    const int gy = max_items < 256 ? 256 : (max_items < 4096 ? max_items : 4096);                             \
    hipLaunchKernelGGL((pa::la::mfma_kernel<R, P, CT>), dim3(gx, gy), dim3(64 * pa::la::NW), lds, st, A);     \
    hipLaunchKernelGGL((pa::la::merge_kernel<R>), dim3(16, std::min(gy, 256)), dim3(256), 0, st, A);           \
    return (int)hipGetLastError();                                                                            \
  } while (0)
    switch (RT) {
#define PA_X(N) case N: if (PT == 0) PA_LA(N, 0); else if (PT == 1) PA_LA(N, 1); else PA_LA(N, 2); break;
      PA_LA_RT(PA_X)
#undef PA_X
      default: break;
    }
#undef PA_LA
  }
  if (Rp > 2048 || D * 4 + 2048 > 64 * 1024) return -2;
  const dim3 grid(H, max_items < 4096 ? max_items : 4096);
  const int lds = (D + 256 + 4) * 4;
  if (fp32) hipLaunchKernelGGL((pa::la::simple_kernel<float>), grid, dim3(256), lds, st, A);
  else hipLaunchKernelGGL((pa::la::simple_kernel<pa::bf16>), grid, dim3(256), lds, st, A);
  return (int)hipGetLastError();
}
