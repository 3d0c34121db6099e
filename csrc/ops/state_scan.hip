// State-space recurrence (Mamba-2) for decode rows and prompt portions of a ragged step, with a causal
// convolution ahead of it. Per head h (group g = h / (H / G)):
//
//   u = silu(conv(x | B | C)),   dt = softplus(dt_raw + bias)
//   S <- exp(-a dt) S + dt B x^T,   y = S^T C + D x
//
// State of a sequence (its slot): S fp32 [H, V, N], N innermost, and the convolution's inputs in a ring:
// the input of position p in row p % RING. A sequence whose portion starts at position 0 starts from
// zeros whatever its slot holds, so a slot is handed on without being cleared.
//
// Projection rows [z: H V | x: H V | B: G N | C: G N | dt: H], V padded to 16 and N to 32 per head and
// group; xBC channels Cc = H V + 2 G N in that order.
//
// Short portions (at most `scan_min` tokens, decode rows among them): step_kernel, convolution included,
// token after token; the ring has room for their inputs beside the taps they read.
// Longer ones (bf16), in chunks of 64 tokens (the scheduler's scan items):
//   conv_kernel   u for all their rows
//   chunk_state   U_c = sum_j exp(L - l_j) dt_j B_j x_j^T          l = running sum of -a dt, L = its end
//   state_pass    S_c = state before chunk c, in place of U_c; the last one to the slot
//   chunk_out     y_i = exp(l_i) C_i . S_c + sum_{j <= i} exp(l_i - l_j) dt_j (C_i . B_j) x_j + D x_i
// The MFMA operands are bf16. B, C and x are bf16 values; everything that carries a decay, a step size or
// the state goes in as a pair of bf16 (value and remainder), 16 bits of mantissa: the recurrence keeps
// the accuracy of fp32 to that order, and chunked and stepped portions agree.
// fp32 models: conv_kernel and step_kernel for long portions too.
#include "common.h"

#include <algorithm>

namespace pa {
namespace ss {

constexpr int LC = 64;        // tokens of a chunk
constexpr int LD = LC + 8;    // LDS row of a chunk's tokens, in elements
constexpr int MAX_SHORT = 8;  // tokens of a short portion at most

struct Args {
  const void* proj;        // [T, ldp]
  void* u;                 // [T, Cc] convolved rows of long portions
  void* y;                 // [T, ldy] (columns h * V + v)
  float* state;            // [slots, H, V, N]
  void* ring;              // [slots, RING, Cc]
  float* work;             // [items, H, V, N]
  float* total;            // [items, H]: a chunk's summed log decay
  const void* conv_w;      // [taps, Cc] fp32, oldest first
  const float *conv_b, *dt_bias, *a, *d;
  const int *q_start, *q_len, *ctx_len, *state_slot, *scan_first;
  const int4* items;
  const int* n_items;
  int ldp, ldy, H, G, V, N, Cc, taps, RING, scan_min, max_seqs, long_too, vsplit;
};

template <typename T>
__device__ __forceinline__ float ld(const void* p, size_t i) { return (float)((const T*)p)[i]; }
__device__ __forceinline__ float silu(float x) { return x / (1.f + __expf(-x)); }
__device__ __forceinline__ float softplus(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

// value and remainder
__device__ __forceinline__ void split(float x, bf16& hi, bf16& lo) {
  hi = (bf16)x;
  lo = (bf16)(x - (float)hi);
}

// ---- convolution of long portions: 8 channels x 16 tokens a thread ---------------------------------
template <typename T, int TAPS>
__global__ __launch_bounds__(256) void conv_kernel(const Args A) {
  const int c8 = (blockIdx.x * 64 + (threadIdx.x & 63)) * 8, sub = threadIdx.x >> 6;
  if (c8 >= A.Cc) return;
  const int inner = A.H * A.V;
  const float* W = (const float*)A.conv_w;
  float w[TAPS][8], b[8];
#pragma unroll
  for (int k = 0; k < TAPS; ++k)
#pragma unroll
    for (int j = 0; j < 8; ++j) w[k][j] = W[(size_t)k * A.Cc + c8 + j];
#pragma unroll
  for (int j = 0; j < 8; ++j) b[j] = A.conv_b[c8 + j];
  const int n_items = A.n_items[0];
  for (int item = blockIdx.y; item < n_items; item += gridDim.y) {
    const int4 it = A.items[item];
    const int s = it.x, t0 = it.y + sub * 16, t1 = min(it.y + it.z, t0 + 16);
    if (t0 >= t1) continue;
    const int q0 = A.q_start[s], p0 = A.ctx_len[s] - A.q_len[s];
    const T* ring = (const T*)A.ring + (size_t)A.state_slot[s] * A.RING * A.Cc + c8;
    auto load = [&](int t, float (&v)[8]) {  // input of the portion's token t (negative: before it)
      T a[8];
      if (t >= 0) {
        __builtin_memcpy(a, __builtin_assume_aligned((const T*)A.proj + (size_t)(q0 + t) * A.ldp + inner + c8, sizeof(T) * 8), sizeof(T) * 8);
      } else if (p0 + t >= 0) {
        __builtin_memcpy(a, __builtin_assume_aligned(ring + (size_t)((p0 + t) % A.RING) * A.Cc, sizeof(T) * 8), sizeof(T) * 8);
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j) a[j] = (T)0.f;
      }
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] = (float)a[j];
    };
    float x[TAPS][8];
#pragma unroll
    for (int k = 0; k < TAPS - 1; ++k) load(t0 - (TAPS - 1) + k, x[k + 1]);
    T* out = (T*)A.u + (size_t)q0 * A.Cc + c8;
#pragma unroll 4
    for (int t = t0; t < t1; ++t) {
#pragma unroll
      for (int k = 0; k + 1 < TAPS; ++k)
#pragma unroll
        for (int j = 0; j < 8; ++j) x[k][j] = x[k + 1][j];
      load(t, x[TAPS - 1]);
      T o[8];
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        float v = b[j];
#pragma unroll
        for (int k = 0; k < TAPS; ++k) v = fmaf(w[k][j], x[k][j], v);
        o[j] = (T)silu(v);
      }
      __builtin_memcpy(__builtin_assume_aligned(out + (size_t)t * A.Cc, sizeof(T) * 8), o, sizeof(T) * 8);
    }
  }
}

// Channels [c0, c1) of the last `rows` positions of a long portion go to the ring: nobody reads it any
// more in this step (the convolution was a launch of its own).
template <typename T>
__device__ __forceinline__ void store_ring(const Args& A, int s, int c0, int c1) {
  const int q0 = A.q_start[s], n = A.q_len[s], p0 = A.ctx_len[s] - n, inner = A.H * A.V, rows = min(A.taps - 1, n);
  T* ring = (T*)A.ring + (size_t)A.state_slot[s] * A.RING * A.Cc;
  for (int e = threadIdx.x; e < rows * (c1 - c0); e += blockDim.x) {
    const int i = e / (c1 - c0), c = c0 + e - i * (c1 - c0), t = n - rows + i;
    ring[(size_t)((p0 + t) % A.RING) * A.Cc + c] = ((const T*)A.proj)[(size_t)(q0 + t) * A.ldp + inner + c];
  }
}

// ---- token by token: a workgroup per (sequence, head, part of V) -------------------------------------
constexpr int REGS = 8;  // state vectors of a thread that stay in registers over the portion

// TN: N / 4 as a constant (8 .. 64) where the state fits the registers of the workgroup; 0: any sizes.
template <typename T, int TAPS, int TN>
__global__ __launch_bounds__(256, 4) void step_kernel(const Args A) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int h = blockIdx.x / A.vsplit, vpart = blockIdx.x % A.vsplit, s = blockIdx.y;
  const int n = A.q_len[s];
  if (n <= 0 || A.state_slot[s] < 0) return;
  const bool conv = n <= A.scan_min;  // short: the convolution is done here
  if (!conv && !A.long_too) return;
  const int V = A.V, N = TN ? 4 * TN : A.N, g = h / (A.H / A.G), inner = A.H * V;
  float *sB = sm, *sC = sm + N, *sx = sm + 2 * N, *sdt = sm + 2 * N + V;  // one token
  const int q0 = A.q_start[s], p0 = A.ctx_len[s] - n;
  float* S = A.state + ((size_t)A.state_slot[s] * A.H + h) * V * N;
  T* ring = (T*)A.ring + (size_t)A.state_slot[s] * A.RING * A.Cc;
  const float* W = (const float*)A.conv_w;
  // lanes along N, 4 values each (a power of two of them, whole groups inside a wave), the rest along V
  int tn = TN ? TN : 1;
  if constexpr (TN == 0)
    while (tn < 64 && (N >> 2) % (2 * tn) == 0) tn *= 2;
  const int ln = threadIdx.x % tn, lv = threadIdx.x / tn, nv = 256 / tn;
  const int v0 = vpart * (V / A.vsplit), v1 = v0 + V / A.vsplit;
  const float a = A.a[h], dd = A.d[h], bias = A.dt_bias[h];
  // the state in registers over the portion: a lane's vectors are of rows v0 + lv + k nv
  f32x4 st[TN ? REGS : 1];
  float* mine = S + (size_t)(v0 + lv) * N + 4 * ln;
  if constexpr (TN > 0) {
#pragma unroll
    for (int k = 0; k < REGS; ++k) {
      st[k] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (p0 > 0 && v0 + lv + k * nv < v1) st[k] = *reinterpret_cast<const f32x4*>(mine + (size_t)k * nv * N);
    }
  }
  for (int t = 0; t < n; ++t) {
    const T* row = (const T*)A.proj + (size_t)(q0 + t) * A.ldp;
    __syncthreads();
    for (int e = threadIdx.x; e < 2 * N + v1 - v0; e += 256) {
      const int c = e < N ? inner + g * N + e : e < 2 * N ? inner + A.G * N + g * N + e - N : h * V + v0 + e - 2 * N;
      float v;
      if (conv) {
        v = A.conv_b[c];
        float x[TAPS];
#pragma unroll
        for (int k = 0; k < TAPS; ++k) {
          const int i = t - (TAPS - 1) + k;
          x[k] = 0.f;
          if (i >= 0) x[k] = (float)((const T*)A.proj)[(size_t)(q0 + i) * A.ldp + inner + c];
          else if (p0 + i >= 0) x[k] = (float)ring[(size_t)((p0 + i) % A.RING) * A.Cc + c];
        }
#pragma unroll
        for (int k = 0; k < TAPS; ++k) v = fmaf(W[(size_t)k * A.Cc + c], x[k], v);
        v = (float)(T)silu(v);
        // the owner of a channel keeps its input (rows that no token of this portion reads)
        if (e >= 2 * N || (h % (A.H / A.G) == 0 && vpart == 0)) ring[(size_t)((p0 + t) % A.RING) * A.Cc + c] = row[inner + c];
      } else {
        v = (float)((const T*)A.u)[(size_t)(q0 + t) * A.Cc + c];
      }
      if (e < 2 * N) sm[e] = v;
      else sx[v0 + e - 2 * N] = v;
    }
    if (threadIdx.x == 255) {  // (a thread of the last wave, which has the fewest channels)
      const float dt = softplus((float)row[inner + A.Cc + h] + bias);
      sdt[0] = dt;
      sdt[1] = expf(-a * dt);
    }
    __syncthreads();
    const float dt = sdt[0], decay = sdt[1];
    // one vector's step; returns its part of S^T C
    auto step = [&](f32x4& w, int i, float u) {
      const f32x4 b = *reinterpret_cast<const f32x4*>(sB + i), c = *reinterpret_cast<const f32x4*>(sC + i);
      float acc = 0.f;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        w[j] = w[j] * decay + u * b[j];
        acc = fmaf(w[j], c[j], acc);
      }
      return acc;
    };
    auto finish = [&](float acc, int v, float x) {
#pragma unroll
      for (int o = 32; o > 0; o >>= 1)
        if (tn > o) acc += __shfl_xor(acc, o, 64);
      if (ln == 0) ((T*)A.y)[(size_t)(q0 + t) * A.ldy + h * V + v] = (T)(acc + dd * x);
    };
    if constexpr (TN > 0) {
#pragma unroll
      for (int k = 0; k < REGS; ++k) {
        const int v = v0 + lv + k * nv;
        if (v < v1) {
          const float x = sx[v];
          finish(step(st[k], 4 * ln, dt * x), v, x);
        }
      }
    } else {
      const bool fresh = p0 + t == 0;
      for (int v = v0 + lv; v < v1; v += nv) {
        const float x = sx[v];
        float acc = 0.f;
        for (int i = ln * 4; i < N; i += tn * 4) {
          f32x4* p = reinterpret_cast<f32x4*>(S + (size_t)v * N + i);
          f32x4 w = fresh ? f32x4{0.f, 0.f, 0.f, 0.f} : *p;
          acc += step(w, i, dt * x);
          *p = w;
        }
        finish(acc, v, x);
      }
    }
  }
  if constexpr (TN > 0) {
#pragma unroll
    for (int k = 0; k < REGS; ++k)
      if (v0 + lv + k * nv < v1) *reinterpret_cast<f32x4*>(mine + (size_t)k * nv * N) = st[k];
  }
  if (!conv && vpart == 0) {
    const int per = (A.Cc + A.H - 1) / A.H;
    store_ring<T>(A, s, min(A.Cc, h * per), min(A.Cc, (h + 1) * per));
  }
}

// ---- chunks -------------------------------------------------------------------------------------------
// Loads come first and together: a chunk's work is short against their latency.
// A token's raw step size (wave 0), rows past the end whatever the last one has
__device__ __forceinline__ float load_dt(const Args& A, int h, int row0, int n) {
  if (threadIdx.x >= 64) return 0.f;
  return (float)((const bf16*)A.proj)[(size_t)(row0 + min((int)threadIdx.x, n - 1)) * A.ldp + A.H * A.V + A.Cc + h] + A.dt_bias[h];
}
// dt and the running log decay of a chunk's tokens (wave 0), rows past the end neutral
__device__ __forceinline__ void chunk_steps(const Args& A, int h, float raw, int n, float* dt, float* l) {
  if (threadIdx.x < 64) {
    const int j = threadIdx.x;
    const float d = j < n ? softplus(raw) : 0.f;
    float x = -A.a[h] * d;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float y = __shfl_up(x, o, 64);
      if (j >= o) x += y;
    }
    dt[j] = d;
    l[j] = x;
  }
}
// 8 columns of one of a chunk's rows (unit e of D / 8 columns x 64 rows); rows past the end repeat the
// last one, and meet weights of 0
__device__ __forceinline__ bf16x8 load_cols(const bf16* u, int ld, int e, int D, int n) {
  return *reinterpret_cast<const bf16x8*>(u + (size_t)min(e & (LC - 1), n - 1) * ld + min((e >> 6) * 8, D - 8));
}
constexpr int XB = 2, BB = 4, SB = 8;  // units of x, B and the state that a thread loads ahead

__global__ __launch_bounds__(256) void chunk_state_kernel(const Args A) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int h = blockIdx.x, n_items = A.n_items[0];
  const int V = A.V, N = A.N, g = h / (A.H / A.G), inner = A.H * V;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, lg = lane >> 4, c = lane & 15;
  float *dt = (float*)smem, *l = dt + LC;
  bf16* bt = (bf16*)(smem + 2 * LC * 4);  // [N][LD]: B transposed
  bf16 *xh = bt + N * LD, *xl = xh + V * LD;  // [V][LD]: weighted x transposed, value and remainder
  for (int item = blockIdx.y; item < n_items; item += gridDim.y) {
    const int4 it = A.items[item];
    const int n = it.z, row0 = A.q_start[it.x] + it.y;
    const bf16 *ux = (const bf16*)A.u + (size_t)row0 * A.Cc + h * V, *ub = (const bf16*)A.u + (size_t)row0 * A.Cc + inner + g * N;
    const float raw = load_dt(A, h, row0, n);
    bf16x8 xv[XB], bv[BB];
#pragma unroll
    for (int i = 0; i < BB; ++i) bv[i] = load_cols(ub, A.Cc, threadIdx.x + 256 * i, N, n);
#pragma unroll
    for (int i = 0; i < XB; ++i) xv[i] = load_cols(ux, A.Cc, threadIdx.x + 256 * i, V, n);
    __syncthreads();
    chunk_steps(A, h, raw, n, dt, l);
    auto put_b = [&](int e, const bf16x8& b) {
      const int j = e & (LC - 1), i = (e >> 6) * 8;
      if (i >= N) return;
#pragma unroll
      for (int k = 0; k < 8; ++k) bt[(i + k) * LD + j] = b[k];
    };
#pragma unroll
    for (int i = 0; i < BB; ++i) put_b(threadIdx.x + 256 * i, bv[i]);
    for (int e = threadIdx.x + 256 * BB; e < (N >> 3) * LC; e += 256) put_b(e, load_cols(ub, A.Cc, e, N, n));
    __syncthreads();
    const float end = l[LC - 1];
    auto put_x = [&](int e, const bf16x8& x) {
      const int j = e & (LC - 1), i = (e >> 6) * 8;
      if (i >= V) return;
      const float w = j < n ? dt[j] * expf(end - l[j]) : 0.f;
#pragma unroll
      for (int k = 0; k < 8; ++k) {
        bf16 hi, lo;
        split(w * (float)x[k], hi, lo);
        xh[(i + k) * LD + j] = hi;
        xl[(i + k) * LD + j] = lo;
      }
    };
#pragma unroll
    for (int i = 0; i < XB; ++i) put_x(threadIdx.x + 256 * i, xv[i]);
    for (int e = threadIdx.x + 256 * XB; e < (V >> 3) * LC; e += 256) put_x(e, load_cols(ux, A.Cc, e, V, n));
    __syncthreads();
    float* out = A.work + ((size_t)item * A.H + h) * V * N;
    const int tn = N >> 4, tv = V >> 4;
    for (int t = wid; t < tn * tv; t += 4) {
      const int n0 = (t % tn) * 16, v0 = (t / tn) * 16;
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const bf16x8 b = *reinterpret_cast<const bf16x8*>(bt + (n0 + c) * LD + 32 * k + 8 * lg);
        const bf16x8 x0 = *reinterpret_cast<const bf16x8*>(xh + (v0 + c) * LD + 32 * k + 8 * lg);
        const bf16x8 x1 = *reinterpret_cast<const bf16x8*>(xl + (v0 + c) * LD + 32 * k + 8 * lg);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(b, x0, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(b, x1, acc, 0, 0, 0);
      }
      *reinterpret_cast<f32x4*>(out + (size_t)(v0 + c) * N + n0 + 4 * lg) = acc;
    }
    if (threadIdx.x == 0) A.total[(size_t)item * A.H + h] = end;
  }
}

// 4 state values a thread, chunk after chunk; the next 8 chunks are on their way while 8 are written
__global__ __launch_bounds__(256) void state_pass_kernel(const Args A) {
  const int h = blockIdx.z, VN = A.V * A.N, e = (blockIdx.x * 256 + threadIdx.x) * 4, n_items = A.n_items[0];
  if (e >= VN) return;
  const size_t step = (size_t)A.H * VN;
  for (int item = blockIdx.y; item < n_items; item += gridDim.y) {
    const int4 it = A.items[item];
    if (it.y != 0) continue;  // a portion's first item takes all of them
    const int s = it.x, n = A.q_len[s], chunks = (n + LC - 1) / LC;
    float* S = A.state + ((size_t)A.state_slot[s] * A.H + h) * VN + e;
    f32x4 st = {0.f, 0.f, 0.f, 0.f};
    if (A.ctx_len[s] > n) st = *reinterpret_cast<const f32x4*>(S);
    float* w = A.work + ((size_t)item * A.H + h) * VN + e;
    const float* tot = A.total + (size_t)item * A.H + h;
    f32x4 u[8], un[8];
    float d[8], dn[8];
    auto load = [&](int c0, f32x4 (&uu)[8], float (&ddd)[8]) {
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int k = min(c0 + i, chunks - 1);
        uu[i] = *reinterpret_cast<const f32x4*>(w + k * step);
        ddd[i] = tot[(size_t)k * A.H];
      }
    };
    load(0, u, d);
    for (int c0 = 0; c0 < chunks; c0 += 8) {
      if (c0 + 8 < chunks) load(c0 + 8, un, dn);
#pragma unroll
      for (int i = 0; i < 8; ++i)
        if (c0 + i < chunks) {
          *reinterpret_cast<f32x4*>(w + (c0 + i) * step) = st;
          const float f = expf(d[i]);
#pragma unroll
          for (int j = 0; j < 4; ++j) st[j] = st[j] * f + u[i][j];
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

// STAGED: the incoming state is split into LDS once; otherwise every wave reads it from memory.
// NK: N / 32 as a constant, for which C stays in registers and B's loads go out together; 0: any N.
template <bool STAGED, int NK>
__global__ __launch_bounds__(256) void chunk_out_kernel(const Args A) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int h = blockIdx.x, n_items = A.n_items[0];
  const int V = A.V, N = NK ? 32 * NK : A.N, g = h / (A.H / A.G), inner = A.H * V, NL = N + 8;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, lg = lane >> 4, c = lane & 15;
  float *dt = (float*)smem, *l = dt + LC;
  bf16 *mh = (bf16*)(smem + 2 * LC * 4), *ml = mh + LC * LD;  // [i][LD], value and remainder
  bf16* xt = ml + LC * LD;                                    // [V][LD]
  bf16 *sh = xt + V * LD, *sl = sh + V * NL;                  // [V][NL], value and remainder
  for (int item = blockIdx.y; item < n_items; item += gridDim.y) {
    const int4 it = A.items[item];
    const int n = it.z, row0 = A.q_start[it.x] + it.y;
    const bf16* u = (const bf16*)A.u + (size_t)row0 * A.Cc;
    const float* S = A.work + ((size_t)item * A.H + h) * V * N;
    // (rows past the end repeat the last one; their results are dropped)
    const int i = 16 * wid + c, ri = min(i, n - 1);
    const bf16* cr = u + (size_t)ri * A.Cc + inner + A.G * N + g * N + 8 * lg;
    const bf16* ux = u + h * V;
    const float raw = load_dt(A, h, row0, n);
    bf16x8 cf[NK ? NK : 1], xv[XB];
    f32x4 cb[4];  // C_i . B_j
    f32x4 sv[STAGED ? SB : 1];
#pragma unroll
    for (int k = 0; k < XB; ++k) xv[k] = load_cols(ux, A.Cc, threadIdx.x + 256 * k, V, n);
    auto load_state = [&](int e) { return *reinterpret_cast<const f32x4*>(S + min(e, V * N - 4)); };
    if constexpr (STAGED) {
#pragma unroll
      for (int k = 0; k < SB; ++k) sv[k] = load_state(1024 * k + threadIdx.x * 4);
    }
    if constexpr (NK > 0) {
#pragma unroll
      for (int k = 0; k < NK; ++k) cf[k] = *reinterpret_cast<const bf16x8*>(cr + 32 * k);
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) {
        cb[jt] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (jt <= wid) {
          const bf16* br = u + (size_t)min(16 * jt + c, n - 1) * A.Cc + inner + g * N + 8 * lg;
          bf16x8 bf[NK ? NK : 1];
#pragma unroll
          for (int k = 0; k < NK; ++k) bf[k] = *reinterpret_cast<const bf16x8*>(br + 32 * k);
#pragma unroll
          for (int k = 0; k < NK; ++k) cb[jt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf[k], cf[k], cb[jt], 0, 0, 0);
        }
      }
    }
    __syncthreads();
    chunk_steps(A, h, raw, n, dt, l);
    auto put_x = [&](int e, const bf16x8& x) {
      const int j = e & (LC - 1), i = (e >> 6) * 8;
      if (i >= V) return;
#pragma unroll
      for (int k = 0; k < 8; ++k) xt[(i + k) * LD + j] = x[k];
    };
#pragma unroll
    for (int k = 0; k < XB; ++k) put_x(threadIdx.x + 256 * k, xv[k]);
    for (int e = threadIdx.x + 256 * XB; e < (V >> 3) * LC; e += 256) put_x(e, load_cols(ux, A.Cc, e, V, n));
    if constexpr (STAGED) {
      auto put_state = [&](int e, const f32x4& v) {
        if (e >= V * N) return;
        const int r = e / N, k0 = e - r * N;
        bf16x4 hi, lo;
#pragma unroll
        for (int k = 0; k < 4; ++k) {
          bf16 a, b;
          split(v[k], a, b);
          hi[k] = a;
          lo[k] = b;
        }
        *reinterpret_cast<bf16x4*>(sh + r * NL + k0) = hi;
        *reinterpret_cast<bf16x4*>(sl + r * NL + k0) = lo;
      };
#pragma unroll
      for (int k = 0; k < SB; ++k) put_state(1024 * k + threadIdx.x * 4, sv[k]);
      for (int e = 1024 * SB + threadIdx.x * 4; e < V * N; e += 1024) put_state(e, load_state(e));
    }
    __syncthreads();
    // M[i][j] = exp(l_i - l_j) dt_j (C_i . B_j), a lane's row i, its columns j = 16 jt + 4 lg ..
    const float li = l[i];
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) {
      bf16x4 hi = {(bf16)0.f, (bf16)0.f, (bf16)0.f, (bf16)0.f}, lo = hi;
      if (jt <= wid) {
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
        if constexpr (NK > 0) {
          acc = cb[jt];
        } else {
          const bf16* br = u + (size_t)min(16 * jt + c, n - 1) * A.Cc + inner + g * N + 8 * lg;
          for (int k = 0; k < N; k += 32)
            acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(br + k),
                                                          *reinterpret_cast<const bf16x8*>(cr + k), acc, 0, 0, 0);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int j = 16 * jt + 4 * lg + r;
          bf16 a, b;
          split(j <= i ? acc[r] * (expf(li - l[j]) * dt[j]) : 0.f, a, b);
          hi[r] = a;
          lo[r] = b;
        }
      }
      *reinterpret_cast<bf16x4*>(mh + i * LD + 16 * jt + 4 * lg) = hi;
      *reinterpret_cast<bf16x4*>(ml + i * LD + 16 * jt + 4 * lg) = lo;
    }
    __syncthreads();
    bf16x8 m0[2], m1[2];
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      m0[k] = *reinterpret_cast<const bf16x8*>(mh + i * LD + 32 * k + 8 * lg);
      m1[k] = *reinterpret_cast<const bf16x8*>(ml + i * LD + 32 * k + 8 * lg);
    }
    const float ei = expf(li), dd = A.d[h];
    for (int v0 = 0; v0 < V; v0 += 16) {
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
      auto from_state = [&](int k) {
        bf16x8 s0, s1;
        if (STAGED) {
          s0 = *reinterpret_cast<const bf16x8*>(sh + (v0 + c) * NL + k + 8 * lg);
          s1 = *reinterpret_cast<const bf16x8*>(sl + (v0 + c) * NL + k + 8 * lg);
        } else {
          const float* p = S + (size_t)(v0 + c) * N + k + 8 * lg;
#pragma unroll
          for (int q = 0; q < 8; ++q) {
            bf16 a, b;
            split(p[q], a, b);
            s0[q] = a;
            s1[q] = b;
          }
        }
        const bf16x8 cv = NK ? cf[NK ? k / 32 : 0] : *reinterpret_cast<const bf16x8*>(cr + k);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(s0, cv, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(s1, cv, acc, 0, 0, 0);
      };
      if constexpr (NK > 0) {
#pragma unroll
        for (int k = 0; k < NK; ++k) from_state(32 * k);
      } else {
        for (int k = 0; k < N; k += 32) from_state(k);
      }
      acc *= ei;
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const bf16x8 x = *reinterpret_cast<const bf16x8*>(xt + (v0 + c) * LD + 32 * k + 8 * lg);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(x, m0[k], acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(x, m1[k], acc, 0, 0, 0);
      }
      if (i < n) {
        bf16x4 o;
#pragma unroll
        for (int r = 0; r < 4; ++r) o[r] = (bf16)(acc[r] + dd * (float)xt[(v0 + 4 * lg + r) * LD + i]);
        *reinterpret_cast<bf16x4*>((bf16*)A.y + (size_t)(row0 + i) * A.ldy + h * V + v0 + 4 * lg) = o;
      }
    }
    if (it.y == 0) {  // the portion's first chunk: this head's share of the channels
      const int per = (A.Cc + A.H - 1) / A.H;
      store_ring<bf16>(A, it.x, min(A.Cc, h * per), min(A.Cc, (h + 1) * per));
    }
  }
}

}  // namespace ss
}  // namespace pa

// max_items: room of the scan items; 0 when no portion of this launch can be longer than scan_min
extern "C" int pa_state_scan(int fp32, const void* proj, int ldp, void* u, void* y, int ldy, float* state, void* ring,
                             float* work, float* total, const float* conv_w, const float* conv_b, const float* dt_bias,
                             const float* a, const float* d, const int* q_start, const int* q_len, const int* ctx_len,
                             const int* state_slot, const int* scan_first, const int* items, const int* n_items,
                             int max_items, int seqs, int H, int G, int V, int N, int taps, int ring_rows,
                             int scan_min, hipStream_t st) {
  using namespace pa::ss;
  if (seqs <= 0) return 0;
  if (V % 16 || N % 32 || H % G || scan_min > MAX_SHORT || ring_rows < taps - 1 + scan_min || (taps != 4 && taps != 8)) return -1;  // (shorter ones are padded)
  Args A{proj, u, y, state, ring, work, total, conv_w, conv_b, dt_bias, a, d, q_start, q_len, ctx_len, state_slot,
         scan_first, (const int4*)items, n_items, ldp, ldy, H, G, V, N, H * V + 2 * G * N, taps, ring_rows, scan_min,
         seqs, fp32, 1};
  if (A.Cc % 8 || ldp % 8) return -1;
  if (max_items > 0) {
    const dim3 grid((A.Cc / 8 + 63) / 64, std::min(max_items, 4096));
#define PA_CONV(T)                                                                                        \
  do {                                                                                                    \
    if (taps == 4) hipLaunchKernelGGL((conv_kernel<T, 4>), grid, dim3(256), 0, st, A);                    \
    else hipLaunchKernelGGL((conv_kernel<T, 8>), grid, dim3(256), 0, st, A);                              \
  } while (0)
    if (fp32) PA_CONV(float); else PA_CONV(pa::bf16);
#undef PA_CONV
  }
  // few sequences: a head's V over more workgroups
  while (A.vsplit < 8 && H * seqs * A.vsplit < 512 && V % (A.vsplit * 2) == 0) A.vsplit *= 2;
  const int step_lds = (2 * N + V + 2) * 4;
  if (step_lds > 64 * 1024) return -2;
  const dim3 sgrid(H * A.vsplit, seqs);
  const int tn = V / A.vsplit <= REGS * 1024 / N ? N / 4 : 0;
#define PA_STEP_N(T, K)                                                                                   \
  do {                                                                                                    \
    if (taps == 4) hipLaunchKernelGGL((step_kernel<T, 4, K>), sgrid, dim3(256), step_lds, st, A);         \
    else hipLaunchKernelGGL((step_kernel<T, 8, K>), sgrid, dim3(256), step_lds, st, A);                   \
  } while (0)
#define PA_STEP(T)                                                                                        \
  do {                                                                                                    \
    if (tn == 8) PA_STEP_N(T, 8);                                                                         \
    else if (tn == 16) PA_STEP_N(T, 16);                                                                  \
    else if (tn == 32) PA_STEP_N(T, 32);                                                                  \
    else if (tn == 64) PA_STEP_N(T, 64);                                                                  \
    else PA_STEP_N(T, 0);                                                                                 \
  } while (0)
  if (fp32) PA_STEP(float); else PA_STEP(pa::bf16);
#undef PA_STEP
#undef PA_STEP_N
  if (fp32 || max_items <= 0) return (int)hipGetLastError();
  const int lds_s = 2 * LC * 4 + (N + 2 * V) * LD * 2;
  const int lds_o = 2 * LC * 4 + (2 * LC + V) * LD * 2, staged = lds_o + 2 * V * (N + 8) * 2;
  constexpr int MAX_LDS = 160 * 1024;
  if (lds_s > MAX_LDS || lds_o > MAX_LDS) return -2;
  static bool attr = false;
  if (!attr) {
    (void)hipFuncSetAttribute((const void*)chunk_state_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, MAX_LDS);
    attr = true;
  }
  const dim3 grid(H, std::min(max_items, 4096));
  hipLaunchKernelGGL(chunk_state_kernel, grid, dim3(256), lds_s, st, A);
  hipLaunchKernelGGL(state_pass_kernel, dim3((V * N / 4 + 255) / 256, std::min(max_items, 16), H), dim3(256), 0, st, A);
  const bool in_lds = staged <= 80 * 1024;
  const int lds = in_lds ? staged : lds_o;
#define PA_OUT(S, K)                                                                                                       \
  do {                                                                                                                     \
    static bool set = false;                                                                                               \
    if (!set) {                                                                                                            \
      (void)hipFuncSetAttribute((const void*)chunk_out_kernel<S, K>, hipFuncAttributeMaxDynamicSharedMemorySize, MAX_LDS); \
      set = true;                                                                                                          \
    }                                                                                                                      \
    hipLaunchKernelGGL((chunk_out_kernel<S, K>), grid, dim3(256), lds, st, A);                                             \
  } while (0)
  if (!in_lds) PA_OUT(false, 0);
  else if (N == 32) PA_OUT(true, 1);
  else if (N == 64) PA_OUT(true, 2);
  else if (N == 128) PA_OUT(true, 4);
  else PA_OUT(true, 0);
#undef PA_OUT
  return (int)hipGetLastError();
}
