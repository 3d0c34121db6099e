// Grouped projections: many small weight matrices, each applied to its own rows.
//
//   dense   every row goes through every group, group h reading its own columns of x and writing
//           its own columns of out (per-head up-projections of latent attention)
//   sorted  row p belongs to one group: mixture-of-experts layers, rows sorted by expert into
//           tiles of at most TM rows (table_route_kernel below)
//
// Weights are packed per group like the other projections ([N/16, K/32, 64, 8], one 16-B lane
// vector per MFMA operand). The MFMA's A operand is W and its B operand x, so a lane's four
// accumulators are four consecutive outputs of one row: 8-byte stores, and the gated pair
// (tiles 2i: gate, 2i + 1: up) is lane-local. Tiles of 16 rows stream the weights (decode steps); 64
// rows share them; prompts with 256 rows and more per group run the ping-pong kernels instead
// (gemm_prefill.hip pa_expert_tiles).
//
// Epilogues: plain, the gated unit of packed_epi.h (limit, alpha, cubic, bias), or the square of relu; of dense rows
// also the product times sigmoid(gate), and the gated unit whose second factor is the row's embedding in a table.
// Sorted rows may have weights: the product is that of weight * x.
#include "packed_epi.h"

extern "C" int pa_expert_tiles(void* y, const void* x, const void* wp, long long wstride, int N, int K, int ldx, int ldy,
                               const int* tiles, int max_tiles, const int* n_tiles, const int* order, int x_div,
                               int out_order, int epi, float limit, float alpha, float cubic, float bias, const float* row_w,
                               hipStream_t st);

namespace pa {
namespace gg {

struct Args {
  const void* x;
  const void* w;
  void* out;
  long long wstride;       // elements per group
  int ldx, xg, ldo, og;    // row strides and per-group column offsets (dense)
  int rows, N16, K32;      // dense rows; N16 = packed 16-row tiles per group
  const int4* tiles;       // sorted: {group, first position, rows, 0}
  const int* n_tiles;
  const int* order;        // sorted: position -> token * top + k
  int x_div;               // sorted: x row = order / x_div (0: x row = position)
  int out_order;           // sorted: out row = order[position] (0: out row = position)
  float limit, alpha, cubic, bias;
  // dense, optional: after a group's N columns of out, the rotated part of the row's head (r columns of
  // x at the group's offset + rskip, the first rd turned by the row's position), padded to rp columns
  const int* positions;
  const float* cos_sin;
  int rskip, r, rp, rd;
  int wide;  // out rows and group offsets are multiples of 8 elements
  const float* row_w;      // sorted, optional: by order[position], the weight of x's row
  // dense, optional: gate [rows, ldg], columns as out's; table rows ids[row], its columns at tcol as out's
  const void *gate, *table;
  const int* ids;
  int ldg, ldt, tcol, vocab;
};

// The rotated columns of `n` rows from `start` of group grp (one workgroup).
template <typename T>
__device__ __forceinline__ void rotate_rows(const Args& A, int grp, int start, int n) {
  const int half = A.rd >> 1, N = A.N16 * 16;
  if (sizeof(T) == 2 && half % 8 == 0 && A.rd == A.r && A.rskip % 8 == 0 && A.xg % 8 == 0 && A.og % 8 == 0 &&
      A.ldo % 8 == 0) {
    // 8 pairs a thread, 16-byte accesses
    const int hp = half >> 3;
    for (int e = threadIdx.x; e < n * hp; e += 256) {
      const int t = start + e / hp, j = (e % hp) * 8;
      const bf16* src = (const bf16*)A.x + (size_t)t * A.ldx + (size_t)grp * A.xg + A.rskip + j;
      bf16* dst = (bf16*)A.out + (size_t)t * A.ldo + (size_t)grp * A.og + N + j;
      const float* cs = A.cos_sin + (size_t)A.positions[t] * A.rd + j;
      const bf16x8 u = *reinterpret_cast<const bf16x8*>(src), v = *reinterpret_cast<const bf16x8*>(src + half);
      float c[8], s[8];
      __builtin_memcpy(c, cs, 32);
      __builtin_memcpy(s, cs + half, 32);
      bf16x8 a, b;
#pragma unroll
      for (int k = 0; k < 8; ++k) {
        a[k] = (bf16)((float)u[k] * c[k] - (float)v[k] * s[k]);
        b[k] = (bf16)((float)v[k] * c[k] + (float)u[k] * s[k]);
      }
      *reinterpret_cast<bf16x8*>(dst) = a;
      *reinterpret_cast<bf16x8*>(dst + half) = b;
    }
    for (int e = threadIdx.x; e < n * (A.rp - A.r); e += 256)
      ((T*)A.out)[(size_t)(start + e / (A.rp - A.r)) * A.ldo + (size_t)grp * A.og + N + A.r + e % (A.rp - A.r)] = (T)0.f;
    return;
  }
  const int per = max(1, 256 / A.rp), i0 = threadIdx.x / A.rp;  // rows at a time
  for (int j = threadIdx.x % A.rp; j < A.rp && i0 < per; j += 256) {
#pragma unroll 4
    for (int i = i0; i < n; i += per) {
      const int t = start + i;
      const T* src = (const T*)A.x + (size_t)t * A.ldx + (size_t)grp * A.xg + A.rskip;
      float v = 0.f;
      if (j < A.r) {
        v = (float)src[j];
        const float* cs = A.cos_sin + (size_t)A.positions[t] * A.rd;
        if (j < half) v = v * cs[j] - (float)src[j + half] * cs[half + j];
        else if (j < A.rd) v = v * cs[j - half] + (float)src[j - half] * cs[j];
      }
      ((T*)A.out)[(size_t)t * A.ldo + (size_t)grp * A.og + N + j] = (T)v;
    }
  }
}

__device__ __forceinline__ float glu(float g, float u, const Args& A) {
  return pk::gated_unit(g, u, A.limit, A.alpha, A.cubic, A.bias);
}

enum { PLAIN = 0, GLU = 1, RELU2 = 2, GATED = 3, TABLE = 4 };

// where the second factor of a dense row's outputs lies (GATED, TABLE)
template <typename T, int EPI>
__device__ __forceinline__ const T* factor_row(const Args& A, int row, int grp) {
  if constexpr (EPI == GATED) return (const T*)A.gate + (size_t)row * A.ldg + (size_t)grp * A.og;
  return (const T*)A.table + (size_t)min(max(A.ids[row], 0), A.vocab - 1) * A.ldt + A.tcol;
}
template <int EPI>
__device__ __forceinline__ float times(float a, float f, const Args& A) {
  if constexpr (EPI == GATED) return a / (1.f + __expf(-f));
  return glu(a, f, A);
}

template <int MT, int NT, int KU, int EPI>
__global__ __launch_bounds__(256) void gemm_kernel(const Args A) {
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int c = lane & 15, g = lane >> 4;
  int grp, start, n;
  if (A.tiles) {
    if ((int)blockIdx.y >= A.n_tiles[0]) return;
    const int4 tl = A.tiles[blockIdx.y];
    grp = tl.x;
    start = tl.y;
    n = tl.z;
  } else {
    grp = blockIdx.z;
    start = blockIdx.y * (16 * MT);
    n = min(16 * MT, A.rows - start);
  }
  if (A.rp && blockIdx.x == 0) {
    rotate_rows<bf16>(A, grp, start, n);
    return;
  }
  const int nt0 = (((int)blockIdx.x - (A.rp ? 1 : 0)) * 4 + wid) * NT;
  if (nt0 >= A.N16) return;
  const bf16* wp = (const bf16*)A.w + (size_t)grp * A.wstride + lane * 8;
  const bf16* wt[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) wt[i] = wp + (size_t)min(nt0 + i, A.N16 - 1) * A.K32 * 512;
  const bf16* xr[MT];
  int pos[MT];
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const int i = min(16 * m + c, n - 1);
    pos[m] = start + i;
    int row = pos[m];
    if (A.tiles && A.x_div) row = A.order[pos[m]] / A.x_div;
    xr[m] = (const bf16*)A.x + (size_t)row * A.ldx + (A.tiles ? 0 : (size_t)grp * A.xg) + 8 * g;
  }
  f32x4 acc[MT][NT];
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int i = 0; i < NT; ++i) acc[m][i] = f32x4{0.f, 0.f, 0.f, 0.f};
  bf16x8 a[KU][NT], b[KU][MT];
  auto load = [&](int s, bf16x8 (&aa)[KU][NT], bf16x8 (&bb)[KU][MT]) {
#pragma unroll
    for (int k = 0; k < KU; ++k) {
#pragma unroll
      for (int i = 0; i < NT; ++i) aa[k][i] = *reinterpret_cast<const bf16x8*>(wt[i] + (size_t)(s + k) * 512);
#pragma unroll
      for (int m = 0; m < MT; ++m) bb[k][m] = *reinterpret_cast<const bf16x8*>(xr[m] + (size_t)(s + k) * 32);
    }
  };
  load(0, a, b);
  for (int s = 0; s < A.K32; s += KU) {
    bf16x8 an[KU][NT], bn[KU][MT];
    if (s + KU < A.K32) load(s + KU, an, bn);
#pragma unroll
    for (int k = 0; k < KU; ++k)
#pragma unroll
      for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int i = 0; i < NT; ++i)
          acc[m][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[k][i], b[k][m], acc[m][i], 0, 0, 0);
#pragma unroll
    for (int k = 0; k < KU; ++k) {
#pragma unroll
      for (int i = 0; i < NT; ++i) a[k][i] = an[k][i];
#pragma unroll
      for (int m = 0; m < MT; ++m) b[k][m] = bn[k][m];
    }
  }
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    if (16 * m + c >= n) continue;
    const int orow = (A.tiles && A.out_order) ? A.order[pos[m]] : pos[m];
    bf16* o = (bf16*)A.out + (size_t)orow * A.ldo + (A.tiles ? 0 : (size_t)grp * A.og) + 4 * g;
    if constexpr (EPI == GLU) {
      const float rw = A.row_w ? A.row_w[A.order[pos[m]]] : 1.f;
#pragma unroll
      for (int i = 0; i + 1 < NT; i += 2) {
        if (nt0 + i >= A.N16) break;
        bf16x4 v;
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] = (bf16)glu(acc[m][i][j] * rw, acc[m][i + 1][j] * rw, A);
        *reinterpret_cast<bf16x4*>(o + (nt0 + i) * 8) = v;
      }
    } else if constexpr (EPI == GATED) {
      const bf16* f = factor_row<bf16, EPI>(A, pos[m], grp) + 4 * g;
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        if (nt0 + i >= A.N16) break;
        const bf16x4 fv = *reinterpret_cast<const bf16x4*>(f + (nt0 + i) * 16);
        bf16x4 v;
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] = (bf16)times<EPI>(acc[m][i][j], (float)fv[j], A);
        *reinterpret_cast<bf16x4*>(o + (nt0 + i) * 16) = v;
      }
    } else if (NT % 2 == 0 && A.N16 % 2 == 0 && A.wide) {
      // 16-byte stores: lanes of neighbouring lane groups trade halves
      const struct { bf16* y; int ldy; } row{o - 4 * g, 0};
#pragma unroll
      for (int i = 0; i + 1 < NT; i += 2) {
        if (nt0 + i >= A.N16) break;
        pk::store_pair_wide<EPI == RELU2 ? pk::EP_RELU2 : pk::EP_PLAIN>(row, 0, nt0 + i, g, acc[m][i], acc[m][i + 1]);
      }
    } else {
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        if (nt0 + i >= A.N16) break;
        bf16x4 v;
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] = (bf16)(EPI == RELU2 ? pk::relu2(acc[m][i][j]) : acc[m][i][j]);
        *reinterpret_cast<bf16x4*>(o + (nt0 + i) * 16) = v;
      }
    }
  }
}

// Dense rows through one group of few outputs (TABLE): 8 waves share a tile of 16 MT rows and 16 NT outputs, each every
// eighth step of K, and add up through LDS.
template <int MT, int NT>
__global__ __launch_bounds__(512) void split_k_kernel(const Args A) {
  extern __shared__ __attribute__((aligned(16))) f32x4 red[];  // [8][MT NT][64]
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, c = lane & 15, g = lane >> 4;
  // tiles of the same rows next to each other on one XCD: they share its copy of x
  const int cols = (A.N16 + NT - 1) / NT, tiles = cols * ((A.rows + 16 * MT - 1) / (16 * MT)), per = (tiles + 7) >> 3;
  const int tile = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
  if ((int)(blockIdx.x >> 3) >= per || tile >= tiles) return;
  const int nt0 = tile % cols * NT, start = tile / cols * (16 * MT), n = min(16 * MT, A.rows - start);
  const bf16 *wt[NT], *xr[MT];
#pragma unroll
  for (int i = 0; i < NT; ++i) wt[i] = (const bf16*)A.w + (size_t)min(nt0 + i, A.N16 - 1) * A.K32 * 512 + lane * 8;
#pragma unroll
  for (int m = 0; m < MT; ++m) xr[m] = (const bf16*)A.x + (size_t)(start + min(16 * m + c, n - 1)) * A.ldx + 8 * g;
  f32x4 acc[MT][NT];
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int i = 0; i < NT; ++i) acc[m][i] = f32x4{0.f, 0.f, 0.f, 0.f};
  constexpr int U = MT * NT == 1 ? 8 : 4;  // steps whose loads go out together
  for (int s = wid; s < A.K32; s += 8 * U) {
    bf16x8 a[U][NT], b[U][MT];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = min(s + 8 * u, A.K32 - 1);
#pragma unroll
      for (int i = 0; i < NT; ++i) a[u][i] = *reinterpret_cast<const bf16x8*>(wt[i] + (size_t)k * 512);
#pragma unroll
      for (int m = 0; m < MT; ++m) b[u][m] = *reinterpret_cast<const bf16x8*>(xr[m] + (size_t)k * 32);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (s + 8 * u < A.K32) {
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
          for (int i = 0; i < NT; ++i) acc[m][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[u][i], b[u][m], acc[m][i], 0, 0, 0);
      }
  }
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int i = 0; i < NT; ++i) red[((wid * MT + m) * NT + i) * 64 + lane] = acc[m][i];
  __syncthreads();
  for (int t = wid; t < MT * NT; t += 8) {  // tile (m, i): the same lanes again
    const int m = t / NT, i = t % NT, row = start + 16 * m + c;
    f32x4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int w = 0; w < 8; ++w) v += red[((w * MT + m) * NT + i) * 64 + lane];
    if (16 * m + c >= n || nt0 + i >= A.N16) continue;
    const int col = (nt0 + i) * 16 + 4 * g;
    const bf16x4 f = *reinterpret_cast<const bf16x4*>(factor_row<bf16, TABLE>(A, row, 0) + col);
    bf16x4 o;
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] = (bf16)times<TABLE>(v[j], (float)f[j], A);
    *reinterpret_cast<bf16x4*>((bf16*)A.out + (size_t)row * A.ldo + col) = o;
  }
}

// fp32: one output (or gated pair) per thread, weights row-major [G, 16 N16, 32 K32] in the same
// row order as the packed ones. The exact path; not tuned.
template <int EPI>
__global__ __launch_bounds__(256) void gemm_f32_kernel(const Args A) {
  constexpr bool PAIR = EPI == GLU;
  constexpr int TM = 16;
  __shared__ float xs[TM][33], w0[16][33], w1[16][33];
  const int tn = threadIdx.x & 15, tm = threadIdx.x >> 4;
  int grp, start, n;
  if (A.tiles) {
    if ((int)blockIdx.y >= A.n_tiles[0]) return;
    const int4 tl = A.tiles[blockIdx.y];
    grp = tl.x; start = tl.y; n = tl.z;
  } else {
    grp = blockIdx.z;
    start = blockIdx.y * TM;
    n = min(TM, A.rows - start);
  }
  if (A.rp && blockIdx.x == 0) {
    rotate_rows<float>(A, grp, start, n);
    return;
  }
  const int bx = (int)blockIdx.x - (A.rp ? 1 : 0);
  const int K = A.K32 * 32;
  const float* wg = (const float*)A.w + (size_t)grp * A.wstride + (size_t)bx * (PAIR ? 32 : 16) * K;
  float a0 = 0.f, a1 = 0.f;
  for (int k0 = 0; k0 < K; k0 += 32) {
    __syncthreads();
    for (int e = threadIdx.x; e < TM * 32; e += 256) {
      const int m = e >> 5, k = e & 31, p = start + min(m, n - 1);
      int row = p;
      if (A.tiles && A.x_div) row = A.order[p] / A.x_div;
      xs[m][k] = ((const float*)A.x)[(size_t)row * A.ldx + (A.tiles ? 0 : (size_t)grp * A.xg) + k0 + k];
      w0[m][k] = wg[(size_t)m * K + k0 + k];
      if (PAIR) w1[m][k] = wg[(size_t)(16 + m) * K + k0 + k];
    }
    __syncthreads();
#pragma unroll 8
    for (int k = 0; k < 32; ++k) {
      a0 += xs[tm][k] * w0[tn][k];
      if (PAIR) a1 += xs[tm][k] * w1[tn][k];
    }
  }
  if (tm >= n) return;
  const int p = start + tm;
  const int orow = (A.tiles && A.out_order) ? A.order[p] : p;
  float* o = (float*)A.out + (size_t)orow * A.ldo + (A.tiles ? 0 : (size_t)grp * A.og) + bx * 16 + tn;
  if constexpr (PAIR) {
    const float rw = A.row_w ? A.row_w[A.order[p]] : 1.f;
    *o = glu(a0 * rw, a1 * rw, A);
  } else if constexpr (EPI == GATED || EPI == TABLE) {
    *o = times<EPI>(a0, factor_row<float, EPI>(A, p, grp)[bx * 16 + tn], A);
  } else {
    *o = EPI == RELU2 ? pk::relu2(a0) : a0;
  }
}

// Routing by token id, for every expert layer of the model in one launch (workgroup = layer):
// layer l's table [vocab, top] (int32, at tables + desc[0]) names the token's experts. Rows with
// slot < 0 (padding) are left out. Writes, at the layer's offsets,
//   order[p] = token * top + k, positions sorted by expert;  tiles: at most tm rows of one expert each.
constexpr int ROUTE_DESC = 8;  // {table offset, vocab, top, experts, order offset, tile offset, max tiles, 0}
constexpr int ROUTE_EMAX = 2048;

__global__ __launch_bounds__(1024) void table_route_kernel(const int* __restrict__ tables, const int* __restrict__ desc,
                                                           const int* __restrict__ ids, const int* __restrict__ slots,
                                                           int T, int tm, int* __restrict__ order,
                                                           int4* __restrict__ tiles, int* __restrict__ n_tiles) {
  __shared__ int cnt[ROUTE_EMAX], base[ROUTE_EMAX], tbase[ROUTE_EMAX], ws[2][16];
  const int* d = desc + blockIdx.x * ROUTE_DESC;
  const int V = d[1], top = d[2], E = d[3];
  const int* tab = tables + d[0];
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  for (int e = threadIdx.x; e < E; e += 1024) cnt[e] = 0;
  __syncthreads();
  auto expert = [&](int p) {
    const int t = p / top;
    if (slots[t] < 0) return -1;
    const int e = tab[(size_t)min(max(ids[t], 0), V - 1) * top + (p - t * top)];
    return min(max(e, 0), E - 1);
  };
  for (int p = threadIdx.x; p < T * top; p += 1024) {
    const int e = expert(p);
    if (e >= 0) atomicAdd(&cnt[e], 1);
  }
  __syncthreads();
  // exclusive scans of the row and tile counts, 1,024 experts at a time
  int carry_r = 0, carry_t = 0;
  for (int e0 = 0; e0 < E; e0 += 1024) {
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
    int or_ = carry_r, oq = carry_t, tr = 0, tq = 0;
    for (int w = 0; w < 16; ++w) {
      if (w < wid) { or_ += ws[0][w]; oq += ws[1][w]; }
      tr += ws[0][w];
      tq += ws[1][w];
    }
    if (e < E) { base[e] = or_ + sr - r; tbase[e] = oq + sq - q; }
    carry_r += tr;
    carry_t += tq;
    __syncthreads();
  }
  int4* tl = tiles + d[5];
  for (int e = threadIdx.x; e < E; e += 1024)
    for (int i = 0, k = tbase[e]; i < cnt[e]; i += tm, ++k)
      if (k < d[6]) tl[k] = int4{e, base[e] + i, min(tm, cnt[e] - i), 0};
  if (threadIdx.x == 0) n_tiles[blockIdx.x] = min(carry_t, d[6]);
  __syncthreads();
  int* ord = order + d[4];
  for (int p = threadIdx.x; p < T * top; p += 1024) {
    const int e = expert(p);
    if (e >= 0) ord[atomicAdd(&base[e], 1)] = p;
  }
}

}  // namespace gg
}  // namespace pa

extern "C" int pa_table_route(const int* tables, const int* desc, int layers, const int* ids, const int* slots, int T,
                              int tm, int* order, int* tiles, int* n_tiles, hipStream_t st) {
  if (layers <= 0 || T <= 0) return 0;
  hipLaunchKernelGGL(pa::gg::table_route_kernel, dim3(layers), dim3(1024), 0, st, tables, desc, ids, slots, T, tm,
                     order, (int4*)tiles, n_tiles);
  return (int)hipGetLastError();
}

// tm: rows per sorted tile (16, 64 or 256; dense: the kernel's choice by row count)
extern "C" int pa_grouped_gemm(int fp32, const void* x, const void* w, void* out, long long wstride, int groups,
                               int ldx, int xg, int ldo, int og, int rows, int N16, int K32, const int* tiles,
                               int max_tiles, const int* n_tiles, const int* order, int x_div, int out_order, int tm,
                               int epi, float limit, float alpha, float cubic, float bias, const int* positions,
                               const float* cos_sin, int rskip, int r, int rp, int rd, const float* row_w, const void* gate,
                               int ldg, const void* table, const int* ids, int ldt, int tcol, int vocab, hipStream_t st) {
  if (N16 <= 0 || K32 <= 0 || (epi == 1 && N16 % 2)) return -1;
  if (row_w && (!tiles || epi != 1 || !x_div)) return -1;
  if (tiles ? epi > 2 : (epi == 3 && !gate) || (epi == 4 && (!table || !ids))) return -1;
  if (tiles ? max_tiles <= 0 : rows <= 0) return 0;
  const pa::gg::Args A{x, w, out, wstride, ldx, xg, ldo, og, rows, N16, K32, (const int4*)tiles, n_tiles,
                       order, x_div, out_order, limit, alpha, cubic, bias, positions, cos_sin, rskip, r, rp, rd,
                       ldo % 8 == 0 && og % 8 == 0 && ((uintptr_t)out & 15) == 0, row_w, gate, table, ids, ldg, ldt, tcol, vocab};
  const int rot = rp > 0 ? 1 : 0;  // one more column of workgroups
  if (fp32) {
    if (tiles && tm != 16) return -2;
    const dim3 grid((epi == 1 ? N16 / 2 : N16) + rot, tiles ? max_tiles : (rows + 15) / 16, tiles ? 1 : groups);
    if (epi == 1) hipLaunchKernelGGL((pa::gg::gemm_f32_kernel<pa::gg::GLU>), grid, dim3(256), 0, st, A);
    else if (epi == 2) hipLaunchKernelGGL((pa::gg::gemm_f32_kernel<pa::gg::RELU2>), grid, dim3(256), 0, st, A);
    else if (epi == 3) hipLaunchKernelGGL((pa::gg::gemm_f32_kernel<pa::gg::GATED>), grid, dim3(256), 0, st, A);
    else if (epi == 4) hipLaunchKernelGGL((pa::gg::gemm_f32_kernel<pa::gg::TABLE>), grid, dim3(256), 0, st, A);
    else hipLaunchKernelGGL((pa::gg::gemm_f32_kernel<pa::gg::PLAIN>), grid, dim3(256), 0, st, A);
    return (int)hipGetLastError();
  }
  if (tiles && tm == 256)
    return pa_expert_tiles(out, x, w, wstride, N16 * 16, K32 * 32, ldx, ldo, tiles, max_tiles, n_tiles, order, x_div,
                           out_order, epi == 1 ? pa::pk::EP_GLU : epi == 2 ? pa::pk::EP_RELU2 : pa::pk::EP_PLAIN, limit, alpha, cubic, bias, row_w, st);
  if (epi == 4) {  // tiles as large as leave most of the chip busy
#define PA_SK(MT, NT)                                                                                                       \
  do {                                                                                                                      \
    constexpr int lds = 8 * MT * NT * 1024;                                                                                 \
    static bool attr = false;                                                                                               \
    if (!attr) {                                                                                                            \
      (void)hipFuncSetAttribute((const void*)pa::gg::split_k_kernel<MT, NT>, hipFuncAttributeMaxDynamicSharedMemorySize, lds); \
      attr = true;                                                                                                          \
    }                                                                                                                       \
    hipLaunchKernelGGL((pa::gg::split_k_kernel<MT, NT>), dim3(((N16 + NT - 1) / NT * ((rows + 16 * MT - 1) / (16 * MT)) + 7) / 8 * 8), \
                       dim3(512), lds, st, A);                                                                              \
  } while (0)
    auto fills = [&](int t) { return (N16 + t - 1) / t * ((rows + 16 * t - 1) / (16 * t)) >= 192; };
    if (groups != 1) return -1;
    if (fills(4)) PA_SK(4, 4);
    else if (fills(2)) PA_SK(2, 2);
    else PA_SK(1, 1);
#undef PA_SK
    return (int)hipGetLastError();
  }
  // dense: 64-row tiles once they fill the chip
  if (!tiles) tm = (N16 + 15) / 16 * ((rows + 63) / 64) * groups < 256 ? 16 : 64;
  if (tm != 16 && tm != 64) return -2;
#define PA_GG(MT, NT, KU, G)                                                                                   \
  hipLaunchKernelGGL((pa::gg::gemm_kernel<MT, NT, KU, G>),                                                     \
                     dim3((N16 + 4 * NT - 1) / (4 * NT) + rot, tiles ? max_tiles : (rows + 16 * MT - 1) / (16 * MT), \
                          tiles ? 1 : groups),                                                                 \
                     dim3(256), 0, st, A)
#define PA_GGK(MT, NT, G)                      \
  do {                                         \
    if (K32 % 4 == 0) PA_GG(MT, NT, 4, G);     \
    else if (K32 % 2 == 0) PA_GG(MT, NT, 2, G);\
    else PA_GG(MT, NT, 1, G);                  \
  } while (0)
  if (tm == 16) {
    if (epi == 1) PA_GGK(1, 2, pa::gg::GLU);
    else if (epi == 2) PA_GGK(1, 1, pa::gg::RELU2);
    else if (epi == 3) PA_GGK(1, 1, pa::gg::GATED);
    else PA_GGK(1, 1, pa::gg::PLAIN);
  } else {
    if (epi == 1) PA_GG(4, 4, 1, pa::gg::GLU);
    else if (epi == 2) PA_GG(4, 4, 1, pa::gg::RELU2);
    else if (epi == 3) PA_GG(4, 4, 1, pa::gg::GATED);
    else PA_GG(4, 4, 1, pa::gg::PLAIN);
  }
#undef PA_GGK
#undef PA_GG
  return (int)hipGetLastError();
}
