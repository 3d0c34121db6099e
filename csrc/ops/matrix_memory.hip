// Matrix memory (mLSTM) for decode rows and prompt portions of a ragged step. Per head, with log gates
//
//   i = cap tanh((z_i + b_i) / cap),   f = logsigmoid(cap tanh((z_f + b_f) / cap))
//   m' = max(f + m, i),   S' = e^(f + m - m') S + e^(i - m') k v^T,   n' likewise with k alone
//   o = S'^T q,   div = max(|n' . q|, e^-m') + 1e-6          (q scaled; o / div is the output, gated_norm divides)
//
// State of a sequence (its slot): S fp32 [H, V, N], N innermost. Row vdim of V is n: the value there is 1, so keys are
// summed by the same arithmetic. m is kept at every row ([H, V]): workgroups that share a head read and write their
// own copies. A sequence whose portion starts at position 0 starts from zeros whatever its slot holds.
//
// Projection rows: q [H N] at cq, k at ck, v [H vin] at cv, z_i [H] at ci, z_f behind it. N is padded to 32, vin to 16
// and V to 16 above vdim + 1.
//
// Short portions (at most `scan_min` tokens, decode rows among them), and all of fp32 models: step_kernel, token after
// token. Longer ones (bf16), in chunks of 64 tokens (the scheduler's scan items). With l the running sum of f in a
// chunk, L its end, g_j = i_j - l_j and m_0 the maximum before the chunk, m_t = l_t + M_t, M_t = max(m_0, g_1 .. g_t):
//   chunk_state   U = sum_j e^(g_j - Mc) k_j v_j^T, Mc the largest g
//   memory_pass   S_c, m_c = state before chunk c, in place of U; behind it M = max(m_c, Mc), S <- e^(m_c - M) S_c +
//                 e^(Mc - M) U, m <- L + M; the last one to the slot
//   chunk_out     o_t = e^(m_c - M_t) S_c q_t + sum_{j <= t} e^(g_j - M_t) (k_j . q_t) v_j, n . q alike
// No exponent is positive. The MFMA operands are bf16: q, k and v are bf16 values; what carries a gate or the state goes
// in as a pair of bf16 (value and remainder), so chunked and stepped portions agree to fp32's order.
#include "common.h"

#include <algorithm>

namespace pa {
namespace mm {

constexpr int LC = 64;        // tokens of a chunk
constexpr int LD = LC + 8;    // LDS row of a chunk's tokens, in elements
constexpr int MAX_SHORT = 8;  // tokens of a short portion at most
constexpr float NONE = -1.0e30f;

struct Args {
  const void* x;     // [T, ldx]
  void* y;           // [T, ldy] (columns h * vin + v)
  float* div;        // [T, H]
  float* state;      // [slots, H, V, N]
  float* top;        // [slots, H, V]
  float* work;       // [items, H, V, N]
  float* stat;       // [items, H, 4]: L, Mc, m before the chunk
  const float *ib, *fb;
  const int *q_start, *q_len, *ctx_len, *state_slot;
  const int4* items;
  const int* n_items;
  int ldx, ldy, H, V, vin, vdim, N, cq, ck, cv, ci, scan_min, long_too, vrows, vtile;
  float cap, qs;
};

__device__ __forceinline__ float input_gate(const Args& A, float z) { return A.cap * tanhf(z / A.cap); }
__device__ __forceinline__ float forget_gate(const Args& A, float z) {
  z = A.cap * tanhf(z / A.cap);
  return fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
}
// value and remainder
__device__ __forceinline__ void split(float x, bf16& hi, bf16& lo) {
  hi = (bf16)x;
  lo = (bf16)(x - (float)hi);
}

// ---- token by token: a workgroup per (sequence, head, rows of V) --------------------------------------
constexpr int REGS = 8;  // state vectors of a thread that stay in registers over the portion

// TN: N / 4 as a constant (8 .. 64) where the state fits the registers of the workgroup; 0: any sizes.
template <typename T, int TN>
__global__ __launch_bounds__(256, 4) void step_kernel(const Args A) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int parts = (A.vdim + A.vrows) / A.vrows;  // rows 0 .. vdim
  const int h = blockIdx.x / parts, v0 = (blockIdx.x % parts) * A.vrows, v1 = min(v0 + A.vrows, A.vdim + 1), s = blockIdx.y;
  const int n = A.q_len[s], slot = A.state_slot[s];
  if (n <= 0 || slot < 0 || (n > A.scan_min && !A.long_too)) return;
  const int N = TN ? 4 * TN : A.N;
  float *sq = sm, *sk = sm + N, *sv = sm + 2 * N, *sg = sv + A.vrows;  // one token
  const int q0 = A.q_start[s], p0 = A.ctx_len[s] - n;
  float* S = A.state + ((size_t)slot * A.H + h) * A.V * N;
  float* top = A.top + ((size_t)slot * A.H + h) * A.V;
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
  float m = p0 > 0 ? top[v0] : 0.f;  // (written behind the token loop's barriers)
  const T* col = (const T*)A.x + (size_t)q0 * A.ldx;
  for (int t = 0; t < n; ++t, col += A.ldx) {
    __syncthreads();
    for (int e = threadIdx.x; e < 2 * N + v1 - v0; e += 256) {
      const int v = v0 + e - 2 * N;
      if (e < 2 * N) sm[e] = (float)col[e < N ? A.cq + h * N + e : A.ck + h * N + e - N];
      else sv[e - 2 * N] = v < A.vdim ? (float)col[A.cv + h * A.vin + v] : 1.f;
    }
    if (threadIdx.x == 255) sg[0] = input_gate(A, (float)col[A.ci + h] + A.ib[h]);
    if (threadIdx.x == 191) sg[1] = forget_gate(A, (float)col[A.ci + A.H + h] + A.fb[h]);
    __syncthreads();
    const float mn = fmaxf(sg[1] + m, sg[0]), keep = expf(sg[1] + m - mn), in = expf(sg[0] - mn);
    m = mn;
    // one vector's step; returns its part of S q
    auto step = [&](f32x4& w, int i, float u) {
      const f32x4 k = *reinterpret_cast<const f32x4*>(sk + i), q = *reinterpret_cast<const f32x4*>(sq + i);
      float acc = 0.f;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        w[j] = w[j] * keep + u * k[j];
        acc = fmaf(w[j], q[j], acc);
      }
      return acc;
    };
    auto finish = [&](float acc, int v) {
#pragma unroll
      for (int o = 32; o > 0; o >>= 1)
        if (tn > o) acc += __shfl_xor(acc, o, 64);
      if (ln != 0) return;
      acc *= A.qs;
      if (v < A.vdim) ((T*)A.y)[(size_t)(q0 + t) * A.ldy + h * A.vin + v] = (T)acc;
      else A.div[(size_t)(q0 + t) * A.H + h] = fmaxf(fabsf(acc), expf(-m)) + 1e-6f;
    };
    if constexpr (TN > 0) {
#pragma unroll
      for (int k = 0; k < REGS; ++k) {
        const int v = v0 + lv + k * nv;
        if (v < v1) finish(step(st[k], 4 * ln, in * sv[v - v0]), v);
      }
    } else {
      const bool fresh = p0 + t == 0;
      for (int v = v0 + lv; v < v1; v += nv) {
        float acc = 0.f;
        for (int i = ln * 4; i < N; i += tn * 4) {
          f32x4* p = reinterpret_cast<f32x4*>(S + (size_t)v * N + i);
          f32x4 w = fresh ? f32x4{0.f, 0.f, 0.f, 0.f} : *p;
          acc += step(w, i, in * sv[v - v0]);
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
  for (int v = v0 + threadIdx.x; v < v1; v += 256) top[v] = m;
}

// ---- chunks -------------------------------------------------------------------------------------------
// A token's raw gates (wave 0), rows past the end whatever the last one has
__device__ __forceinline__ float2 load_gates(const Args& A, int h, int row0, int n) {
  if (threadIdx.x >= 64) return float2{0.f, 0.f};
  const bf16* r = (const bf16*)A.x + (size_t)(row0 + min((int)threadIdx.x, n - 1)) * A.ldx + A.ci + h;
  return float2{(float)r[0] + A.ib[h], (float)r[A.H] + A.fb[h]};
}
// Of a chunk's tokens (wave 0): l, g and the running maximum of g, rows past the end neutral
__device__ __forceinline__ void chunk_gates(const Args& A, float2 raw, int n, float* l, float* g, float* mx) {
  if (threadIdx.x < 64) {
    const int j = threadIdx.x;
    float x = j < n ? forget_gate(A, raw.y) : 0.f;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float y = __shfl_up(x, o, 64);
      if (j >= o) x += y;
    }
    const float gj = j < n ? input_gate(A, raw.x) - x : NONE;
    float top = gj;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float y = __shfl_up(top, o, 64);
      if (j >= o) top = fmaxf(top, y);
    }
    l[j] = x;
    g[j] = gj;
    mx[j] = top;
  }
}
// 8 columns of one of a chunk's rows (unit e of D / 8 columns x 64 rows); rows past the end repeat the last one, and
// meet weights of 0
__device__ __forceinline__ bf16x8 load_cols(const bf16* u, int ld, int e, int D, int n) {
  return *reinterpret_cast<const bf16x8*>(u + (size_t)min(e & (LC - 1), n - 1) * ld + min((e >> 6) * 8, D - 8));
}
// values 8 i .. of a head, from column v on: the projection's, then the row of ones and zeros
__device__ __forceinline__ bf16x8 load_value(const Args& A, const bf16* u, int e, int v0, int n) {
  const int v = v0 + (e >> 6) * 8;
  bf16x8 x = *reinterpret_cast<const bf16x8*>(u + (size_t)min(e & (LC - 1), n - 1) * A.ldx + min(v, A.vin - 8));
  if (v + 8 > A.vdim) {
#pragma unroll
    for (int k = 0; k < 8; ++k)
      if (v + k >= A.vdim) x[k] = (bf16)(v + k == A.vdim ? 1.f : 0.f);
  }
  return x;
}
constexpr int VB = 2, KB = 4, SB = 8;  // units of v, k and the state that a thread loads ahead

__global__ __launch_bounds__(256) void chunk_state_kernel(const Args A) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int tiles = (A.V + A.vtile - 1) / A.vtile, h = blockIdx.x / tiles, v0 = (blockIdx.x % tiles) * A.vtile;
  const int n_items = A.n_items[0], V = min(A.vtile, A.V - v0), N = A.N;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, lg = lane >> 4, c = lane & 15;
  float *l = (float*)smem, *g = l + LC, *mx = g + LC;
  bf16* kt = (bf16*)(smem + 3 * LC * 4);                // [N][LD]: k transposed
  bf16 *vh = kt + N * LD, *vl = vh + A.vtile * LD;      // [vtile][LD]: weighted v transposed, value and remainder
  for (int item = blockIdx.y; item < n_items; item += gridDim.y) {
    const int4 it = A.items[item];
    const int n = it.z, row0 = A.q_start[it.x] + it.y;
    const bf16* x = (const bf16*)A.x + (size_t)row0 * A.ldx;
    const bf16 *xk = x + A.ck + h * N, *xv = x + A.cv + h * A.vin;
    const float2 raw = load_gates(A, h, row0, n);
    bf16x8 vv[VB], kv[KB];
#pragma unroll
    for (int i = 0; i < KB; ++i) kv[i] = load_cols(xk, A.ldx, threadIdx.x + 256 * i, N, n);
#pragma unroll
    for (int i = 0; i < VB; ++i) vv[i] = load_value(A, xv, threadIdx.x + 256 * i, v0, n);
    __syncthreads();
    chunk_gates(A, raw, n, l, g, mx);
    auto put_k = [&](int e, const bf16x8& b) {
      const int j = e & (LC - 1), i = (e >> 6) * 8;
      if (i >= N) return;
#pragma unroll
      for (int k = 0; k < 8; ++k) kt[(i + k) * LD + j] = b[k];
    };
#pragma unroll
    for (int i = 0; i < KB; ++i) put_k(threadIdx.x + 256 * i, kv[i]);
    for (int e = threadIdx.x + 256 * KB; e < (N >> 3) * LC; e += 256) put_k(e, load_cols(xk, A.ldx, e, N, n));
    __syncthreads();
    const float mc = mx[LC - 1];
    auto put_v = [&](int e, const bf16x8& b) {
      const int j = e & (LC - 1), i = (e >> 6) * 8;
      if (i >= V) return;
      const float w = expf(g[j] - mc);
#pragma unroll
      for (int k = 0; k < 8; ++k) {
        bf16 hi, lo;
        split(w * (float)b[k], hi, lo);
        vh[(i + k) * LD + j] = hi;
        vl[(i + k) * LD + j] = lo;
      }
    };
#pragma unroll
    for (int i = 0; i < VB; ++i) put_v(threadIdx.x + 256 * i, vv[i]);
    for (int e = threadIdx.x + 256 * VB; e < (V >> 3) * LC; e += 256) put_v(e, load_value(A, xv, e, v0, n));
    __syncthreads();
    float* out = A.work + (((size_t)item * A.H + h) * A.V + v0) * N;
    const int tn = N >> 4, tv = V >> 4;
    for (int t = wid; t < tn * tv; t += 4) {
      const int n0 = (t % tn) * 16, r0 = (t / tn) * 16;
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const bf16x8 b = *reinterpret_cast<const bf16x8*>(kt + (n0 + c) * LD + 32 * k + 8 * lg);
        const bf16x8 x0 = *reinterpret_cast<const bf16x8*>(vh + (r0 + c) * LD + 32 * k + 8 * lg);
        const bf16x8 x1 = *reinterpret_cast<const bf16x8*>(vl + (r0 + c) * LD + 32 * k + 8 * lg);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(b, x0, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(b, x1, acc, 0, 0, 0);
      }
      *reinterpret_cast<f32x4*>(out + (size_t)(r0 + c) * N + n0 + 4 * lg) = acc;
    }
    if (threadIdx.x == 0 && v0 == 0) {
      float* st = A.stat + ((size_t)item * A.H + h) * 4;
      st[0] = l[LC - 1];
      st[1] = mc;
    }
  }
}

// 4 state values a thread, whole rows a workgroup, chunk after chunk; the next 8 chunks are on their way while 8 are
// written
__global__ __launch_bounds__(256) void memory_pass_kernel(const Args A) {
  const int per = A.N >> 2, rows = max(1, 256 / per), h = blockIdx.z, n_items = A.n_items[0];
  const int r = per <= 256 ? (int)threadIdx.x / per : 0, v = blockIdx.x * rows + r;
  const bool in = r < rows && v < A.V;
  const size_t step = (size_t)A.H * A.V * A.N;
  for (int item = blockIdx.y; item < n_items; item += gridDim.y) {
    const int4 it = A.items[item];
    if (it.y != 0) continue;  // a portion's first item takes all of them
    const int s = it.x, n = A.q_len[s], chunks = (n + LC - 1) / LC;
    const bool fresh = A.ctx_len[s] <= n;
    const size_t head = (size_t)A.state_slot[s] * A.H + h;
    const float m0 = in && !fresh ? A.top[head * A.V + v] : 0.f;
    float mend = m0;
    float* stat = A.stat + ((size_t)item * A.H + h) * 4;
    __syncthreads();  // (a row's maximum is read before its first thread writes it)
    if (in)
      for (int e = ((int)threadIdx.x - r * per) * 4; e < A.N; e += (per <= 256 ? per : 256) * 4) {
        float* S = A.state + (head * A.V + v) * A.N + e;
        f32x4 st = {0.f, 0.f, 0.f, 0.f};
        if (!fresh) st = *reinterpret_cast<const f32x4*>(S);
        float m = m0;
        float* w = A.work + (((size_t)item * A.H + h) * A.V + v) * A.N + e;
        f32x4 u[8], un[8];
        float2 d[8], dn[8];
        auto load = [&](int c0, f32x4 (&uu)[8], float2 (&dd)[8]) {
#pragma unroll
          for (int i = 0; i < 8; ++i) {
            const int k = min(c0 + i, chunks - 1);
            uu[i] = *reinterpret_cast<const f32x4*>(w + k * step);
            dd[i] = *reinterpret_cast<const float2*>(stat + (size_t)k * A.H * 4);
          }
        };
        load(0, u, d);
        for (int c0 = 0; c0 < chunks; c0 += 8) {
          if (c0 + 8 < chunks) load(c0 + 8, un, dn);
#pragma unroll
          for (int i = 0; i < 8; ++i)
            if (c0 + i < chunks) {
              *reinterpret_cast<f32x4*>(w + (c0 + i) * step) = st;
              if (v == 0 && e == 0) stat[(size_t)(c0 + i) * A.H * 4 + 2] = m;
              const float M = fmaxf(m, d[i].y), a = expf(m - M), b = expf(d[i].y - M);
#pragma unroll
              for (int j = 0; j < 4; ++j) st[j] = st[j] * a + u[i][j] * b;
              m = d[i].x + M;
            }
#pragma unroll
          for (int i = 0; i < 8; ++i) {
            u[i] = un[i];
            d[i] = dn[i];
          }
        }
        *reinterpret_cast<f32x4*>(S) = st;
        mend = m;
      }
    if (in && (int)threadIdx.x == r * per) A.top[head * A.V + v] = mend;
  }
}

// NK: N / 32 as a constant, for which q stays in registers and the loads of k go out together; 0: any N.
template <int NK>
__global__ __launch_bounds__(256) void chunk_out_kernel(const Args A) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int tiles = (A.V + A.vtile - 1) / A.vtile, h = blockIdx.x / tiles, vt = (blockIdx.x % tiles) * A.vtile;
  const int n_items = A.n_items[0], V = min(A.vtile, A.V - vt), N = NK ? 32 * NK : A.N, NL = N + 8;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, lg = lane >> 4, c = lane & 15;
  float *l = (float*)smem, *g = l + LC, *mx = g + LC;
  bf16 *mh = (bf16*)(smem + 3 * LC * 4), *ml = mh + LC * LD;  // [i][LD], value and remainder
  bf16* xt = ml + LC * LD;                                    // [vtile][LD]: v transposed
  bf16 *sh = xt + A.vtile * LD, *sl = sh + A.vtile * NL;      // [vtile][NL], value and remainder
  for (int item = blockIdx.y; item < n_items; item += gridDim.y) {
    const int4 it = A.items[item];
    const int n = it.z, row0 = A.q_start[it.x] + it.y;
    const bf16* x = (const bf16*)A.x + (size_t)row0 * A.ldx;
    const float* S = A.work + (((size_t)item * A.H + h) * A.V + vt) * N;
    const float m0 = A.stat[((size_t)item * A.H + h) * 4 + 2];
    // (rows past the end repeat the last one; their results are dropped)
    const int i = 16 * wid + c;
    const bf16 *qr = x + (size_t)min(i, n - 1) * A.ldx + A.cq + h * N + 8 * lg, *xk = x + A.ck + h * N + 8 * lg;
    const bf16* xv = x + A.cv + h * A.vin;
    const float2 raw = load_gates(A, h, row0, n);
    bf16x8 qf[NK ? NK : 1], vv[VB];
    f32x4 kq[4];  // k_j . q_i
    f32x4 sv[SB];
#pragma unroll
    for (int k = 0; k < VB; ++k) vv[k] = load_value(A, xv, threadIdx.x + 256 * k, vt, n);
    auto load_state = [&](int e) { return *reinterpret_cast<const f32x4*>(S + min(e, V * N - 4)); };
#pragma unroll
    for (int k = 0; k < SB; ++k) sv[k] = load_state(1024 * k + threadIdx.x * 4);
    if constexpr (NK > 0) {
#pragma unroll
      for (int k = 0; k < NK; ++k) qf[k] = *reinterpret_cast<const bf16x8*>(qr + 32 * k);
    }
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) {
      kq[jt] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (jt <= wid) {
        const bf16* kr = xk + (size_t)min(16 * jt + c, n - 1) * A.ldx;
        if constexpr (NK > 0) {
          bf16x8 kf[NK ? NK : 1];
#pragma unroll
          for (int k = 0; k < NK; ++k) kf[k] = *reinterpret_cast<const bf16x8*>(kr + 32 * k);
#pragma unroll
          for (int k = 0; k < NK; ++k) kq[jt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[k], qf[k], kq[jt], 0, 0, 0);
        } else {
          for (int k = 0; k < N; k += 32)
            kq[jt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(kr + k),
                                                             *reinterpret_cast<const bf16x8*>(qr + k), kq[jt], 0, 0, 0);
        }
      }
    }
    __syncthreads();
    chunk_gates(A, raw, n, l, g, mx);
    auto put_v = [&](int e, const bf16x8& b) {
      const int j = e & (LC - 1), r = (e >> 6) * 8;
      if (r >= V) return;
#pragma unroll
      for (int k = 0; k < 8; ++k) xt[(r + k) * LD + j] = b[k];
    };
#pragma unroll
    for (int k = 0; k < VB; ++k) put_v(threadIdx.x + 256 * k, vv[k]);
    for (int e = threadIdx.x + 256 * VB; e < (V >> 3) * LC; e += 256) put_v(e, load_value(A, xv, e, vt, n));
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
    __syncthreads();
    // W[i][j] = e^(g_j - M_i) (k_j . q_i), a lane's row i, its columns j = 16 jt + 4 lg ..
    const float M = fmaxf(m0, mx[i]), from = expf(m0 - M);
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) {
      bf16x4 hi = {(bf16)0.f, (bf16)0.f, (bf16)0.f, (bf16)0.f}, lo = hi;
      if (jt <= wid) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int j = 16 * jt + 4 * lg + r;
          bf16 a, b;
          split(j <= i ? kq[jt][r] * expf(g[j] - M) : 0.f, a, b);
          hi[r] = a;
          lo[r] = b;
        }
      }
      *reinterpret_cast<bf16x4*>(mh + i * LD + 16 * jt + 4 * lg) = hi;
      *reinterpret_cast<bf16x4*>(ml + i * LD + 16 * jt + 4 * lg) = lo;
    }
    __syncthreads();
    bf16x8 w0[2], w1[2];
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      w0[k] = *reinterpret_cast<const bf16x8*>(mh + i * LD + 32 * k + 8 * lg);
      w1[k] = *reinterpret_cast<const bf16x8*>(ml + i * LD + 32 * k + 8 * lg);
    }
    for (int r0 = 0; r0 < V; r0 += 16) {
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
      auto from_state = [&](int k) {
        const bf16x8 s0 = *reinterpret_cast<const bf16x8*>(sh + (r0 + c) * NL + k + 8 * lg);
        const bf16x8 s1 = *reinterpret_cast<const bf16x8*>(sl + (r0 + c) * NL + k + 8 * lg);
        const bf16x8 q = NK ? qf[NK ? k / 32 : 0] : *reinterpret_cast<const bf16x8*>(qr + k);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(s0, q, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(s1, q, acc, 0, 0, 0);
      };
      if constexpr (NK > 0) {
#pragma unroll
        for (int k = 0; k < NK; ++k) from_state(32 * k);
      } else {
        for (int k = 0; k < N; k += 32) from_state(k);
      }
      acc *= from;
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const bf16x8 v = *reinterpret_cast<const bf16x8*>(xt + (r0 + c) * LD + 32 * k + 8 * lg);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, w0[k], acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, w1[k], acc, 0, 0, 0);
      }
      if (i < n) {
        acc *= A.qs;
        const int v = vt + r0 + 4 * lg;
        if (v < A.vin) {  // (the column of a padded vdim holds n . q: gated_norm clears it)
          bf16x4 o;
#pragma unroll
          for (int r = 0; r < 4; ++r) o[r] = (bf16)acc[r];
          *reinterpret_cast<bf16x4*>((bf16*)A.y + (size_t)(row0 + i) * A.ldy + h * A.vin + v) = o;
        }
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (v + r == A.vdim) A.div[(size_t)(row0 + i) * A.H + h] = fmaxf(fabsf(acc[r]), expf(-(l[i] + M))) + 1e-6f;
      }
    }
  }
}

}  // namespace mm
}  // namespace pa

// max_items: room of the scan items; 0 when no portion of this launch can be longer than scan_min
extern "C" int pa_matrix_memory(int fp32, const void* x, int ldx, void* y, int ldy, float* div, float* state, float* top,
                                float* work, float* stat, const float* i_bias, const float* f_bias, const int* q_start,
                                const int* q_len, const int* ctx_len, const int* state_slot, const int* items,
                                const int* n_items, int max_items, int seqs, int H, int V, int N, int cq, int ck, int cv,
                                int ci, int vin, int vdim, float cap, float q_scale, int scan_min, hipStream_t st) {
  using namespace pa::mm;
  if (seqs <= 0) return 0;
  if (V % 16 || N % 32 || N <= 0 || vdim < 1 || vin < vdim || vin % 16 || V < vdim + 1 || scan_min > MAX_SHORT || cap <= 0.f ||
      ldx % 8 || ldy % 4 || cq % 8 || ck % 8 || cv % 8) return -1;
  Args A{x, y, div, state, top, work, stat, i_bias, f_bias, q_start, q_len, ctx_len, state_slot, (const int4*)items, n_items,
         ldx, ldy, H, V, vin, vdim, N, cq, ck, cv, ci, scan_min, fp32, 0, 0, cap, q_scale};
  // rows of a workgroup: what its registers hold, fewer where there are few sequences
  const int tn = N == 32 || N == 64 || N == 128 || N == 256 ? N / 4 : 0, pass = tn ? 256 / tn : 16;
  int vrows = tn ? REGS * pass : 64;
  while (vrows > pass && H * seqs * ((vdim + vrows) / vrows) < 512) vrows /= 2;
  const int parts = (vdim + vrows) / vrows;
  A.vrows = std::min(vrows, ((vdim + parts) / parts + pass - 1) / pass * pass);  // (even shares)
  const int step_lds = (2 * N + A.vrows + 2) * 4;
  if (step_lds > 64 * 1024) return -2;
  const dim3 sgrid(H * ((vdim + A.vrows) / A.vrows), seqs);
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
  // rows of V in a chunk's workgroup: two workgroups a CU
  constexpr int MAX_LDS = 160 * 1024;
  auto out_lds = [&](int vt) { return 3 * LC * 4 + (2 * LC + vt) * LD * 2 + 2 * vt * (N + 8) * 2; };
  auto state_lds = [&](int vt) { return 3 * LC * 4 + (N + 2 * vt) * LD * 2; };
  A.vtile = std::min(64, V);
  while (A.vtile > 16 && std::max(out_lds(A.vtile), state_lds(A.vtile)) > MAX_LDS / 2) A.vtile -= 16;
  const int lds_s = state_lds(A.vtile), lds_o = out_lds(A.vtile);
  if (lds_s > MAX_LDS || lds_o > MAX_LDS) return -2;
  const dim3 grid(H * ((V + A.vtile - 1) / A.vtile), std::min(max_items, 4096));
#define PA_ATTR(F)                                                                                       \
  do {                                                                                                   \
    static bool set = false;                                                                             \
    if (!set) {                                                                                          \
      (void)hipFuncSetAttribute((const void*)F, hipFuncAttributeMaxDynamicSharedMemorySize, MAX_LDS);    \
      set = true;                                                                                        \
    }                                                                                                    \
  } while (0)
  PA_ATTR(chunk_state_kernel);
  hipLaunchKernelGGL(chunk_state_kernel, grid, dim3(256), lds_s, st, A);
  const int rows = std::max(1, 1024 / N);
  hipLaunchKernelGGL(memory_pass_kernel, dim3((V + rows - 1) / rows, std::min(max_items, 16), H), dim3(256), 0, st, A);
#define PA_OUT(K)                                                             \
  do {                                                                        \
    PA_ATTR(chunk_out_kernel<K>);                                             \
    hipLaunchKernelGGL(chunk_out_kernel<K>, grid, dim3(256), lds_o, st, A);   \
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
