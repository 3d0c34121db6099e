// Gated linear attention for decode rows and prompt portions of a ragged step. Per head, a decay for every key channel:
//
//   g = logsigmoid(W_a2 a + b) / tau,   S <- diag(e^g) S + k v^T,   o = S^T q          (a: low-rank inputs; q scaled)
//
// State of a sequence (its slot): S fp32 [H, V, N], N innermost. A sequence whose portion starts at position 0 starts
// from zeros whatever its slot holds, so a slot is handed on without being cleared.
//
// Projection rows: q [H N] at cq, k at ck, v [H V] at cv, a [rp] at ca; N is padded to 32 per head, V to 16, a to 32.
//
// Short portions (at most `scan_min` tokens, decode rows among them), and all of fp32 models: step_kernel, token after
// token. Longer ones (bf16), in chunks of 64 tokens (the scheduler's scan items). With l the running sum of g in a
// chunk and L its end (vectors over the channels):
//   prepare       q' = q e^l,  k' = k e^(L - l),  e^L, and the scores A_ij = sum_n q_in k_jn e^(l_in - l_jn), j <= i
//   chunk_state   U = sum_j v_j k'_j^T
//   state_pass    S_c = state before chunk c, in place of U;  S <- S diag(e^L) + U;  the last one to the slot
//   chunk_out     o_i = S_c q'_i + sum_{j <= i} A_ij v_j
// Scores: blocks of 16 x 16 tokens. Behind the diagonal both factors are taken relative to l at the end of the block of
// keys, so no exponent is positive however fast the channels decay; on the diagonal a lane follows its key through the
// block, one decay after the other.
// The MFMA operands are bf16. q, k and v are bf16 values; everything that carries a decay or the state goes in as a pair of
// bf16 (value and remainder), 16 bits of mantissa: chunked and stepped portions agree to that order.
#include "common.h"

#include <algorithm>

namespace pa {
namespace lin {

constexpr int LC = 64;        // tokens of a chunk
constexpr int MAX_SHORT = 8;  // tokens of a short portion at most
constexpr int NT = 128;       // channels of a chunk_state workgroup
typedef __attribute__((address_space(3))) bf16x4 lds_bf16x4;

struct Args {
  const void* x;     // [T, ldx]
  void* y;           // [T, ldy] (columns h * V + v)
  float* state;      // [slots, H, V, N]
  float* work;       // [items, H, V, N]: U, then S_c with every 4 values as 4 + 4 bf16
  bf16 *qd, *kd;     // [2, T, H N]: q', k', values and remainders
  bf16* sc;          // [2, T, H, 64]: scores of a token with its chunk's
  float* end;        // [items, H, N]: e^L
  const void* a2;    // [H N, rp]
  const float* bias; // [H N]
  const int *q_start, *q_len, *ctx_len, *state_slot;
  const int4* items;
  const int* n_items;
  int T, ldx, ldy, H, V, N, rp, cq, ck, cv, ca, scan_min, long_too, vrows, vtile;
  float qs, inv_tau;
};

__device__ __forceinline__ float log_decay(const Args& A, float z) {
  return (fminf(z, 0.f) - log1pf(expf(-fabsf(z)))) * A.inv_tau;
}
// value and remainder
__device__ __forceinline__ void split(float x, bf16& hi, bf16& lo) {
  hi = (bf16)x;
  lo = (bf16)(x - (float)hi);
}
__device__ __forceinline__ void split8(const float (&x)[8], bf16x8& hi, bf16x8& lo) {
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    bf16 a, b;
    split(x[e], a, b);
    hi[e] = a;
    lo[e] = b;
  }
}

// ---- token by token: a workgroup per (sequence, head, rows of V) --------------------------------------
constexpr int REGS = 8;  // state vectors of a thread that stay in registers over the portion

// TN: N / 4 as a constant (8 .. 64) where the state fits the registers of the workgroup; 0: any sizes.
template <typename T, int TN>
__global__ __launch_bounds__(256, 4) void step_kernel(const Args A) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int parts = (A.V + A.vrows - 1) / A.vrows;
  const int h = blockIdx.x / parts, v0 = (blockIdx.x % parts) * A.vrows, v1 = min(v0 + A.vrows, A.V), s = blockIdx.y;
  const int n = A.q_len[s], slot = A.state_slot[s];
  if (n <= 0 || slot < 0 || (n > A.scan_min && !A.long_too)) return;
  const int N = TN ? 4 * TN : A.N;
  float *sq = sm, *sk = sm + N, *sa = sm + 2 * N, *sv = sm + 3 * N;  // one token
  const int q0 = A.q_start[s], p0 = A.ctx_len[s] - n;
  float* S = A.state + ((size_t)slot * A.H + h) * A.V * N;
  int tn = TN ? TN : 1;
  if constexpr (TN == 0)
    while (tn < 64 && (N >> 2) % (2 * tn) == 0) tn *= 2;
  const int ln = threadIdx.x % tn, lv = threadIdx.x / tn, nv = 256 / tn;
  f32x4 st[TN ? REGS : 1];
  float* mine = S + (size_t)(v0 + lv) * N + 4 * ln;
  if constexpr (TN > 0) {
#pragma unroll
    for (int k = 0; k < REGS; ++k) {
      st[k] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (p0 > 0 && v0 + lv + k * nv < v1) st[k] = *reinterpret_cast<const f32x4*>(mine + (size_t)k * nv * N);
    }
  }
  const T* col = (const T*)A.x + (size_t)q0 * A.ldx;
  for (int t = 0; t < n; ++t, col += A.ldx) {
    __syncthreads();
    for (int e = threadIdx.x; e < N; e += 256) {
      const T *w = (const T*)A.a2 + (size_t)(h * N + e) * A.rp, *a = col + A.ca;
      float z = A.bias[h * N + e];
#pragma unroll 4
      for (int r = 0; r < A.rp; r += 8) {
        T wv[8], av[8];
        __builtin_memcpy(wv, __builtin_assume_aligned(w + r, 16), sizeof(wv));
        __builtin_memcpy(av, __builtin_assume_aligned(a + r, 16), sizeof(av));
#pragma unroll
        for (int j = 0; j < 8; ++j) z = fmaf((float)wv[j], (float)av[j], z);
      }
      sa[e] = expf(log_decay(A, z));
    }
    for (int e = threadIdx.x; e < 2 * N + v1 - v0; e += 256) {
      const float v = (float)col[e < N ? A.cq + h * N + e : e < 2 * N ? A.ck + h * N + e - N : A.cv + h * A.V + v0 + e - 2 * N];
      if (e < 2 * N) sm[e] = v;
      else sv[e - 2 * N] = v;
    }
    __syncthreads();
    // one vector's step; returns its part of S q
    auto step = [&](f32x4& w, int i, float u) {
      const f32x4 k = *reinterpret_cast<const f32x4*>(sk + i), q = *reinterpret_cast<const f32x4*>(sq + i);
      const f32x4 d = *reinterpret_cast<const f32x4*>(sa + i);
      float acc = 0.f;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        w[j] = w[j] * d[j] + u * k[j];
        acc = fmaf(w[j], q[j], acc);
      }
      return acc;
    };
    auto finish = [&](float acc, int v) {
#pragma unroll
      for (int o = 32; o > 0; o >>= 1)
        if (tn > o) acc += __shfl_xor(acc, o, 64);
      if (ln == 0) ((T*)A.y)[(size_t)(q0 + t) * A.ldy + h * A.V + v] = (T)(acc * A.qs);
    };
    if constexpr (TN > 0) {
#pragma unroll
      for (int k = 0; k < REGS; ++k) {
        const int v = v0 + lv + k * nv;
        if (v < v1) finish(step(st[k], 4 * ln, sv[v - v0]), v);
      }
    } else {
      const bool fresh = p0 + t == 0;
      for (int v = v0 + lv; v < v1; v += nv) {
        float acc = 0.f;
        for (int i = ln * 4; i < N; i += tn * 4) {
          f32x4* p = reinterpret_cast<f32x4*>(S + (size_t)v * N + i);
          f32x4 w = fresh ? f32x4{0.f, 0.f, 0.f, 0.f} : *p;
          acc += step(w, i, sv[v - v0]);
          *p = w;
        }
        finish(acc, v);
      }
    }
  }
  if constexpr (TN > 0) {
#pragma unroll
    for (int k = 0; k < REGS; ++k)
      if (v0 + lv + k * nv < v1) *reinterpret_cast<f32x4*>(mine + (size_t)k * nv * N) = st[k];
  }
}

// ---- chunks -------------------------------------------------------------------------------------------
// the value that the lane S places down (DOWN) or up holds, among the 16 lanes of a row; 0 past the row's end
template <int S, bool DOWN>
__device__ __forceinline__ float row_shift(float x) {
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, x), (DOWN ? 0x110 : 0x100) + S, 0xf, 0xf, true));
}

// a value that is to be computed here, and not where it is used
__device__ __forceinline__ void pin(float& x) { asm volatile("" : "+v"(x)); }

// The same without branches, for 64 tokens at once: log(1 + t) of the hardware's logarithm, its series where t is small
__device__ __forceinline__ float log_decay_fast(const Args& A, float z) {
  const float t = __expf(-fabsf(z)), series = t * fmaf(t, fmaf(t, fmaf(t, -0.25f, 1.f / 3.f), -0.5f), 1.f);
  float log = __logf(1.f + t);
  pin(log);  // (no branch)
  return (fminf(z, 0.f) - (t < 0.01f ? series : log)) * A.inv_tau;
}

// 4 waves a part, 16 tokens each; a lane holds token 16 w + c and 8 channels of 32. P parts take every P-th 32 channels. Two
// barriers per 32 channels.
template <int P>
__global__ __launch_bounds__(256 * P, 2) void prepare_kernel(const Args A) {
  constexpr int KL = 40;  // LDS row of 32 channels
  __shared__ __attribute__((aligned(16))) bf16 kts[P][2][2][48][KL];  // [turn][value, remainder]: keys to the end of their block
  __shared__ float tots[P][2][4][32];                                  // [turn]: a wave's sum of g
  __shared__ float dg[P][4][16][17];
  __shared__ f32x4 others[P > 1 ? P - 1 : 1][4][3][64];
  const int h = blockIdx.x, n_items = A.n_items[0], N = A.N;
  const int lane = threadIdx.x & 63, wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int part = wid >> 2, w = wid & 3, lg = lane >> 4, c = lane & 15, i = 16 * w + c;
  auto &kt = kts[part];
  auto &tot = tots[part];
  const size_t HN = (size_t)A.H * N, plane = (size_t)A.T * HN;
  const float past[3] = {w > 0 ? 1.f : 0.f, w > 1 ? 1.f : 0.f, w > 2 ? 1.f : 0.f};
  for (int item = blockIdx.y; item < n_items; item += gridDim.y) {
    const int4 it = A.items[item];
    const int n = it.z, row0 = A.q_start[it.x] + it.y, row = row0 + min(i, n - 1);
    const bool live = i < n;
    const float on = live ? 1.f : 0.f;
    const bf16 *xr = (const bf16*)A.x + (size_t)row * A.ldx, *xq = xr + A.cq + h * N + 8 * lg, *xk = xr + A.ck + h * N + 8 * lg;
    const bf16* xa = xr + A.ca + 8 * lg;
    const size_t out = (size_t)row * HN + h * N + 8 * lg;
    const bf16x8 a0 = *reinterpret_cast<const bf16x8*>(xa);
    f32x4 blk[3];
    float d[16];
#pragma unroll
    for (int a = 0; a < 3; ++a) blk[a] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < 16; ++s) d[s] = 0.f;
    // the next channels are on their way: q, k, W_a2's first 32 columns, the bias
    bf16x8 qn, kn, wn[2];
    f32x4 bn[2];
    const bf16* wr = (const bf16*)A.a2 + (size_t)(h * N + 8 * (c >> 2) + (c & 3)) * A.rp + 8 * lg;
    const float* br = A.bias + h * N + 8 * lg;
    auto load = [&](int m) {
      qn = *reinterpret_cast<const bf16x8*>(xq + 32 * m);
      kn = *reinterpret_cast<const bf16x8*>(xk + 32 * m);
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        wn[half] = *reinterpret_cast<const bf16x8*>(wr + (size_t)(32 * m + 4 * half) * A.rp);
        bn[half] = *reinterpret_cast<const f32x4*>(br + 32 * m + 4 * half);
      }
    };
    load(part);
    for (int m = part, turn = 0; m < N / 32; m += P, turn ^= 1) {  // (all parts take as many: N / 32 is a multiple of P)
      const bf16x8 qb = qn, kb = kn, wb[2] = {wn[0], wn[1]};
      const f32x4 bb[2] = {bn[0], bn[1]};
      if (m + P < N / 32) load(m + P);
      // z^T = W_a2 a^T; the rows of W_a2 in the order that gives a lane its 8 channels in two results
      float g[8], q[8], k[8];
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        f32x4 z = bb[half];
        z = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wb[half], a0, z, 0, 0, 0);
        for (int r = 32; r < A.rp; r += 32)
          z = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(wr + (size_t)(32 * m + 4 * half) * A.rp + r),
                                                      *reinterpret_cast<const bf16x8*>(xa + r), z, 0, 0, 0);
#pragma unroll
        for (int r = 0; r < 4; ++r) g[4 * half + r] = log_decay_fast(A, z[r]) * on;
      }
      float l[8], al[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        q[e] = (float)qb[e];
        k[e] = (float)kb[e];
        al[e] = __expf(g[e]);
        float x = g[e];  // running sum over the 16 tokens
        x += row_shift<1, true>(x);
        x += row_shift<2, true>(x);
        x += row_shift<4, true>(x);
        x += row_shift<8, true>(x);
        l[e] = x;
      }
      if (c == 15) {
#pragma unroll
        for (int e = 0; e < 8; ++e) tot[turn][w][8 * lg + e] = l[e];
      }
      __syncthreads();
      // sums up to this wave's block, and of the chunk (the same order of additions everywhere)
      float base[8], L[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float* t = &tot[turn][0][8 * lg + e];
        const float t0 = t[0], t1 = t[32], t2 = t[64];
        base[e] = fmaf(t2, past[2], fmaf(t1, past[1], t0 * past[0]));
        L[e] = t0 + t1 + t2 + t[96];
        pin(base[e]);
        pin(L[e]);
        l[e] += base[e];
      }
      float v[8];
      bf16x8 hi, lo;
      if (w < 3) {
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = k[e] * __expf(base[e] + tot[turn][w][8 * lg + e] - l[e]);
        split8(v, hi, lo);
        *reinterpret_cast<bf16x8*>(&kt[turn][0][i][8 * lg]) = hi;
        *reinterpret_cast<bf16x8*>(&kt[turn][1][i][8 * lg]) = lo;
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = q[e] * A.qs * __expf(l[e]);
      split8(v, hi, lo);
      if (live) {
        *reinterpret_cast<bf16x8*>(A.qd + out + 32 * m) = hi;
        *reinterpret_cast<bf16x8*>(A.qd + plane + out + 32 * m) = lo;
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = k[e] * __expf(L[e] - l[e]);
      split8(v, hi, lo);
      if (live) {
        *reinterpret_cast<bf16x8*>(A.kd + out + 32 * m) = hi;
        *reinterpret_cast<bf16x8*>(A.kd + plane + out + 32 * m) = lo;
      }
      if (i == 0) {
        float* e0 = A.end + ((size_t)item * A.H + h) * N + 32 * m + 8 * lg;
#pragma unroll
        for (int e = 0; e < 8; ++e) e0[e] = __expf(L[e]);
      }
      // the diagonal: lane c follows key c, d[s] += (k_c decayed to c + s) . q_(c+s); queries and decays move up the lanes
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = q[e];
#pragma unroll
      for (int s = 0; s < 16; ++s) {
        if (s > 0) __builtin_amdgcn_sched_barrier(0);  // (all steps' values at once do not fit the registers)
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          if (s > 0) {
            al[e] = row_shift<1, false>(al[e]);
            v[e] = row_shift<1, false>(v[e]);
            k[e] *= al[e];
          }
          d[s] = fmaf(k[e], v[e], d[s]);
        }
        pin(d[s]);
      }
      __syncthreads();
      float R[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};  // l at the end of a block of keys
#pragma unroll
      for (int a = 0; a < 3; ++a)
        if (a < w) {  // wave-uniform
#pragma unroll
          for (int e = 0; e < 8; ++e) {
            R[e] += tot[turn][a][8 * lg + e];
            v[e] = q[e] * A.qs * __expf(l[e] - R[e]);
          }
          split8(v, hi, lo);
          const bf16x8 k0 = *reinterpret_cast<const bf16x8*>(&kt[turn][0][16 * a + c][8 * lg]);
          const bf16x8 k1 = *reinterpret_cast<const bf16x8*>(&kt[turn][1][16 * a + c][8 * lg]);
          blk[a] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k0, hi, blk[a], 0, 0, 0);
          blk[a] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k0, lo, blk[a], 0, 0, 0);
          blk[a] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k1, hi, blk[a], 0, 0, 0);
        }
    }
    // the diagonal's sums over all channels, from a key's lane to the query's row
#pragma unroll
    for (int s = 0; s < 16; ++s) {
      d[s] += __shfl_xor(d[s], 16, 64);
      d[s] += __shfl_xor(d[s], 32, 64);
      if (lg == (s & 3) && c + s < 16) dg[part][w][c + s][c] = d[s] * A.qs;
    }
    if (P > 1 && part > 0) {
#pragma unroll
      for (int a = 0; a < 3; ++a) others[part - 1][w][a][lane] = blk[a];
    }
    __syncthreads();
    if (P > 1 && part == 0) {
#pragma unroll
      for (int o = 0; o < P - 1; ++o)
#pragma unroll
        for (int a = 0; a < 3; ++a) blk[a] += others[o][w][a][lane];
    }
    bf16* o = A.sc + ((size_t)row * A.H + h) * LC + 4 * lg;
    const size_t low = (size_t)A.T * A.H * LC;
#pragma unroll
    for (int a = 0; a < 4; ++a) {
      bf16x4 hi, lo;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        float v = 0.f;
        if (a < 3 && a < w) v = blk[a < 3 ? a : 0][r];
        if (a == w && 4 * lg + r <= c) {
#pragma unroll
          for (int o = 0; o < P; ++o) v += dg[o][w][c][4 * lg + r];
        }
        bf16 x, y;
        split(v, x, y);
        hi[r] = x;
        lo[r] = y;
      }
      if (live && part == 0) {
        *reinterpret_cast<bf16x4*>(o + 16 * a) = hi;
        *reinterpret_cast<bf16x4*>(o + low + 16 * a) = lo;
      }
    }
    __syncthreads();  // (the next item writes dg)
  }
}

// An MFMA operand whose rows are 16 columns of an LDS tile and whose inner index is 32 of its rows (tokens), by two
// transposing reads: lane (c, g) gets column c of tokens 4g .. 4g + 3 and 16 + 4g .. 16 + 4g + 3.
__device__ __forceinline__ bf16x8 columns(const bf16* tile, int ld, int c, int g) {
  const bf16* p = tile + (4 * g + (c >> 2)) * ld + 4 * (c & 3);
  const bf16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds_bf16x4*)p);
  const bf16x4 b = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds_bf16x4*)(p + 16 * ld));
  bf16x8 v;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    v[j] = a[j];
    v[4 + j] = b[j];
  }
  return v;
}

// `cols` (whole 8s) of a chunk's rows into LDS; rows past the end are zero, or repeat the last one
template <bool ZERO>
__device__ __forceinline__ void stage(const bf16* src, size_t ld, int cols, int n, bf16* dst, int ldd) {
  const int units = cols >> 3;
  for (int e = threadIdx.x; e < units * LC; e += 256) {
    const int j = e / units, u = (e - j * units) * 8;
    bf16x8 v = *reinterpret_cast<const bf16x8*>(src + (size_t)min(j, n - 1) * ld + u);
    if (ZERO && j >= n) v = bf16x8{};
    *reinterpret_cast<bf16x8*>(dst + j * ldd + u) = v;
  }
}

__global__ __launch_bounds__(256) void chunk_state_kernel(const Args A) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int vt = (A.V + A.vtile - 1) / A.vtile, nt = (A.N + NT - 1) / NT;
  const int h = blockIdx.x / (vt * nt), rest = blockIdx.x % (vt * nt);
  const int v0 = rest / nt * A.vtile, n0 = rest % nt * NT, V = min(A.vtile, A.V - v0), N = min(NT, A.N - n0);
  const int n_items = A.n_items[0], NL = N + 8, VL = V + 8;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, g = lane >> 4, c = lane & 15;
  bf16 *kh = (bf16*)smem, *kl = kh + LC * NL, *xv = kl + LC * NL;  // [64][NL] twice, [64][VL]
  const size_t HN = (size_t)A.H * A.N, plane = (size_t)A.T * HN;
  for (int item = blockIdx.y; item < n_items; item += gridDim.y) {
    const int4 it = A.items[item];
    const int n = it.z, row0 = A.q_start[it.x] + it.y;
    const bf16* kd = A.kd + (size_t)row0 * HN + h * A.N + n0;
    __syncthreads();
    stage<true>(kd, HN, N, n, kh, NL);
    stage<true>(kd + plane, HN, N, n, kl, NL);
    stage<false>((const bf16*)A.x + (size_t)row0 * A.ldx + A.cv + h * A.V + v0, A.ldx, V, n, xv, VL);
    __syncthreads();
    float* out = A.work + (((size_t)item * A.H + h) * A.V + v0) * A.N + n0;
    const int tn = N >> 4, tv = V >> 4;
    for (int t = wid; t < tn * tv; t += 4) {
      const int nb = (t % tn) * 16, vb = (t / tn) * 16;
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const bf16x8 x = columns(xv + 32 * k * VL + vb, VL, c, g);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(columns(kh + 32 * k * NL + nb, NL, c, g), x, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(columns(kl + 32 * k * NL + nb, NL, c, g), x, acc, 0, 0, 0);
      }
      *reinterpret_cast<f32x4*>(out + (size_t)(vb + c) * A.N + nb + 4 * g) = acc;
    }
  }
}

// 4 state values a thread, chunk after chunk; the next 8 chunks are on their way while 8 are written
__global__ __launch_bounds__(256) void state_pass_kernel(const Args A) {
  const int h = blockIdx.z, VN = A.V * A.N, e = (blockIdx.x * 256 + threadIdx.x) * 4, n_items = A.n_items[0];
  if (e >= VN) return;
  const size_t step = (size_t)A.H * VN, dstep = (size_t)A.H * A.N;
  for (int item = blockIdx.y; item < n_items; item += gridDim.y) {
    const int4 it = A.items[item];
    if (it.y != 0) continue;  // a portion's first item takes all of them
    const int s = it.x, n = A.q_len[s], chunks = (n + LC - 1) / LC;
    float* S = A.state + ((size_t)A.state_slot[s] * A.H + h) * VN + e;
    f32x4 st = {0.f, 0.f, 0.f, 0.f};
    if (A.ctx_len[s] > n) st = *reinterpret_cast<const f32x4*>(S);
    float* w = A.work + ((size_t)item * A.H + h) * VN + e;
    const float* end = A.end + ((size_t)item * A.H + h) * A.N + e % A.N;
    f32x4 u[8], un[8], d[8], dn[8];
    auto load = [&](int c0, f32x4 (&uu)[8], f32x4 (&dd)[8]) {
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int k = min(c0 + i, chunks - 1);
        uu[i] = *reinterpret_cast<const f32x4*>(w + k * step);
        dd[i] = *reinterpret_cast<const f32x4*>(end + k * dstep);
      }
    };
    load(0, u, d);
    for (int c0 = 0; c0 < chunks; c0 += 8) {
      if (c0 + 8 < chunks) load(c0 + 8, un, dn);
#pragma unroll
      for (int i = 0; i < 8; ++i)
        if (c0 + i < chunks) {
          bf16x8 pair;
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            bf16 a, b;
            split(st[j], a, b);
            pair[j] = a;
            pair[4 + j] = b;
            st[j] = st[j] * d[i][j] + u[i][j];
          }
          *reinterpret_cast<bf16x8*>(w + (c0 + i) * step) = pair;
        }
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        u[i] = un[i];
        d[i] = dn[i];
      }
    }
    *reinterpret_cast<f32x4*>(S) = st;
  }
}

// NK: N / 32 as a constant, for which q' stays in registers; 0: any N.
template <int NK>
__global__ __launch_bounds__(256) void chunk_out_kernel(const Args A) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int tiles = (A.V + A.vtile - 1) / A.vtile, h = blockIdx.x / tiles, v0 = (blockIdx.x % tiles) * A.vtile;
  const int n_items = A.n_items[0], V = min(A.vtile, A.V - v0), N = NK ? 32 * NK : A.N, VL = V + 8, SL = N * 4 + 16;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, g = lane >> 4, c = lane & 15, i = 16 * wid + c;
  bf16* xv = (bf16*)smem;            // [64][VL]
  char* ss = smem + LC * VL * 2;     // [V] rows of SL bytes: 4 values, 4 remainders, ..
  const size_t HN = (size_t)A.H * N, plane = (size_t)A.T * HN, low = (size_t)A.T * A.H * LC;
  for (int item = blockIdx.y; item < n_items; item += gridDim.y) {
    const int4 it = A.items[item];
    const int n = it.z, row0 = A.q_start[it.x] + it.y, row = row0 + min(i, n - 1);
    const bf16* qr = A.qd + (size_t)row * HN + h * N + 8 * g;
    bf16x8 qh[NK ? NK : 1], ql[NK ? NK : 1];
    if constexpr (NK > 0) {
#pragma unroll
      for (int k = 0; k < NK; ++k) {
        qh[k] = *reinterpret_cast<const bf16x8*>(qr + 32 * k);
        ql[k] = *reinterpret_cast<const bf16x8*>(qr + plane + 32 * k);
      }
    }
    // the token's scores, in the order of `columns`
    const bf16* ar = A.sc + ((size_t)row * A.H + h) * LC + 4 * g;
    bf16x8 ah[2], al[2];
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      const bf16x4 x0 = *reinterpret_cast<const bf16x4*>(ar + 32 * k), x1 = *reinterpret_cast<const bf16x4*>(ar + 32 * k + 16);
      const bf16x4 y0 = *reinterpret_cast<const bf16x4*>(ar + low + 32 * k), y1 = *reinterpret_cast<const bf16x4*>(ar + low + 32 * k + 16);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        ah[k][j] = x0[j];
        ah[k][4 + j] = x1[j];
        al[k][j] = y0[j];
        al[k][4 + j] = y1[j];
      }
    }
    const char* S = (const char*)(A.work + (((size_t)item * A.H + h) * A.V + v0) * N);
    __syncthreads();
    stage<false>((const bf16*)A.x + (size_t)row0 * A.ldx + A.cv + h * A.V + v0, A.ldx, V, n, xv, VL);
    const int units = N >> 2;  // of 16 bytes in a row
#pragma unroll 8
    for (int e = threadIdx.x; e < V * units; e += 256) {
      const int r = e / units, u = e - r * units;
      *reinterpret_cast<u32x4*>(ss + r * SL + u * 16) = *reinterpret_cast<const u32x4*>(S + (size_t)e * 16);
    }
    __syncthreads();
    for (int r0 = 0; r0 < V; r0 += 16) {
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
      auto from_state = [&](int k, const bf16x8& q0, const bf16x8& q1) {
        const char* p = ss + (r0 + c) * SL + (32 * k + 8 * g) * 4;
        const bf16x8 a = *reinterpret_cast<const bf16x8*>(p), b = *reinterpret_cast<const bf16x8*>(p + 16);
        bf16x8 hi, lo;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          hi[j] = a[j];
          hi[4 + j] = b[j];
          lo[j] = a[4 + j];
          lo[4 + j] = b[4 + j];
        }
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi, q0, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi, q1, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo, q0, acc, 0, 0, 0);
      };
      if constexpr (NK > 0) {
#pragma unroll
        for (int k = 0; k < NK; ++k) from_state(k, qh[k], ql[k]);
      } else {
        for (int k = 0; k < N / 32; ++k)
          from_state(k, *reinterpret_cast<const bf16x8*>(qr + 32 * k), *reinterpret_cast<const bf16x8*>(qr + plane + 32 * k));
      }
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const bf16x8 x = columns(xv + 32 * k * VL + r0, VL, c, g);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(x, ah[k], acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(x, al[k], acc, 0, 0, 0);
      }
      if (i < n) {
        bf16x4 o;
#pragma unroll
        for (int r = 0; r < 4; ++r) o[r] = (bf16)acc[r];
        *reinterpret_cast<bf16x4*>((bf16*)A.y + (size_t)(row0 + i) * A.ldy + h * A.V + v0 + r0 + 4 * g) = o;
      }
    }
  }
}

}  // namespace lin
}  // namespace pa

// max_items: room of the scan items; 0 when no portion of this launch can be longer than scan_min
extern "C" int pa_linear_attention(int fp32, const void* x, int ldx, void* y, int ldy, float* state, float* work, void* qd,
                                   void* kd, void* sc, float* end, const void* a2, const float* bias, const int* q_start,
                                   const int* q_len, const int* ctx_len, const int* state_slot, const int* items,
                                   const int* n_items, int max_items, int seqs, int T, int H, int V, int N, int rp, int cq,
                                   int ck, int cv, int ca, float q_scale, float inv_tau, int scan_min, hipStream_t st) {
  using namespace pa::lin;
  if (seqs <= 0) return 0;
  if (V % 16 || N % 32 || N <= 0 || V <= 0 || rp % 32 || rp <= 0 || scan_min > MAX_SHORT || ldx % 8 || ldy % 4 || cq % 8 || ck % 8 ||
      cv % 8 || ca % 8) return -1;
  Args A{x, y, state, work, (pa::bf16*)qd, (pa::bf16*)kd, (pa::bf16*)sc, end, a2, bias, q_start, q_len, ctx_len, state_slot,
         (const int4*)items, n_items, T, ldx, ldy, H, V, N, rp, cq, ck, cv, ca, scan_min, fp32, 0, 0, q_scale, inv_tau};
  // rows of a workgroup: what its registers hold, fewer where there are few sequences
  const int tn = N == 32 || N == 64 || N == 128 || N == 256 ? N / 4 : 0, pass = tn ? 256 / tn : 16;
  int vrows = tn ? REGS * pass : 64;
  while (vrows > pass && H * seqs * ((V + vrows - 1) / vrows) < 512) vrows /= 2;
  const int parts = (V + vrows - 1) / vrows;
  A.vrows = std::min(vrows, ((V + parts - 1) / parts + pass - 1) / pass * pass);  // (even shares)
  const int step_lds = (3 * N + A.vrows) * 4;
  if (step_lds > 64 * 1024) return -2;
  const dim3 sgrid(H * ((V + A.vrows - 1) / A.vrows), seqs);
#define PA_STEP(T)                                                                                    \
  do {                                                                                                \
    if (tn == 8) hipLaunchKernelGGL((step_kernel<T, 8>), sgrid, dim3(256), step_lds, st, A);          \
    else if (tn == 16) hipLaunchKernelGGL((step_kernel<T, 16>), sgrid, dim3(256), step_lds, st, A);   \
    else if (tn == 32) hipLaunchKernelGGL((step_kernel<T, 32>), sgrid, dim3(256), step_lds, st, A);   \
    else if (tn == 64) hipLaunchKernelGGL((step_kernel<T, 64>), sgrid, dim3(256), step_lds, st, A);   \
    else hipLaunchKernelGGL((step_kernel<T, 0>), sgrid, dim3(256), step_lds, st, A);                  \
  } while (0)
  if (fp32) PA_STEP(float); else PA_STEP(pa::bf16);
#undef PA_STEP
  if (fp32 || max_items <= 0) return (int)hipGetLastError();
  constexpr int MAX_LDS = 160 * 1024;
  const int gy = std::min(max_items, 4096), nt = std::min(N, NT);
  // rows of V in a chunk's workgroup: two workgroups a CU
  auto out_lds = [&](int vt) { return LC * (vt + 8) * 2 + vt * (N * 4 + 16); };
  auto state_lds = [&](int vt) { return 2 * LC * (nt + 8) * 2 + LC * (vt + 8) * 2; };
  A.vtile = std::min(64, V);
  while (A.vtile > 16 && std::max(out_lds(A.vtile), state_lds(A.vtile)) > MAX_LDS / 2) A.vtile -= 16;
  const int lds_s = state_lds(A.vtile), lds_o = out_lds(A.vtile), vts = (V + A.vtile - 1) / A.vtile;
  if (lds_s > MAX_LDS || lds_o > MAX_LDS) return -2;
#define PA_ATTR(F)                                                                                       \
  do {                                                                                                   \
    static bool set = false;                                                                             \
    if (!set) {                                                                                          \
      (void)hipFuncSetAttribute((const void*)F, hipFuncAttributeMaxDynamicSharedMemorySize, MAX_LDS);    \
      set = true;                                                                                        \
    }                                                                                                    \
  } while (0)
  // (few chunks: a head's channels over twice the waves)
  if (N % 64 == 0 && H * gy <= 1024) hipLaunchKernelGGL(prepare_kernel<2>, dim3(H, gy), dim3(512), 0, st, A);
  else hipLaunchKernelGGL(prepare_kernel<1>, dim3(H, gy), dim3(256), 0, st, A);
  PA_ATTR(chunk_state_kernel);
  hipLaunchKernelGGL(chunk_state_kernel, dim3(H * vts * ((N + NT - 1) / NT), gy), dim3(256), lds_s, st, A);
  hipLaunchKernelGGL(state_pass_kernel, dim3((V * N / 4 + 255) / 256, std::min(max_items, 16), H), dim3(256), 0, st, A);
#define PA_OUT(K)                                                                           \
  do {                                                                                      \
    PA_ATTR(chunk_out_kernel<K>);                                                           \
    hipLaunchKernelGGL(chunk_out_kernel<K>, dim3(H * vts, gy), dim3(256), lds_o, st, A);    \
  } while (0)
  if (N == 32) PA_OUT(1);
  else if (N == 64) PA_OUT(2);
  else if (N == 128) PA_OUT(4);
  else if (N == 256) PA_OUT(8);
  else PA_OUT(0);
#undef PA_OUT
#undef PA_ATTR
  return (int)hipGetLastError();
}
