"""Dispatch of the fp32-residual, latent-attention, grouped-projection and gated-linear-attention kernels (modules _latent and
_latent_linear).

Device tensors run the HIP kernels of csrc/ops/{residual_norm, latent_cache, latent_attention,
grouped_gemm, linear_attention, poly_norm}.hip and raise when the module is missing; CPU tensors run the fp32 references of
ops/reference.py. Every function takes its constants as arguments and works in bf16 or fp32.
"""
from __future__ import annotations

from typing import Optional

import torch

from . import reference as ref
from .kernels import _on_gpu, require_family, require_grouped, require_latent

SCAN_CHUNK = 64  # tokens of a scan item of recurrent layers
SCAN_MIN = 8     # longer portions are scanned in chunks
LATENT_TILES = (1, 2, 3, 4, 6, 8, 12, 16)  # latent widths (in 32s) with MFMA kernels (latent_attention.hip)
ROT_TILES = (1, 2)


def pad_to(n: int, m: int) -> int:
    return (n + m - 1) // m * m


def latent_pad(R: int) -> int:
    """Cached width of an R-wide latent: the smallest width with an MFMA kernel, else whole 32s."""
    need = (R + 31) // 32
    return 32 * next((n for n in LATENT_TILES if n >= need), need)


# ---- fp32 residual stream -------------------------------------------------------------------
def residual_norm(resid: torch.Tensor, eps: float, *, y: Optional[torch.Tensor] = None, partials: int = 1,
                  y_scale: float = 1.0, w_post: Optional[torch.Tensor] = None, emb: Optional[torch.Tensor] = None,
                  ids: Optional[torch.Tensor] = None, emb_add: bool = False, w_next: Optional[torch.Tensor] = None,
                  out: Optional[torch.Tensor] = None, rows: Optional[torch.Tensor] = None, post_groups: int = 1,
                  next_groups: int = 1, mix: Optional[torch.Tensor] = None, hist: Optional[torch.Tensor] = None):
    """resid (fp32 [T, D], in place) += norm(y_scale * sum of a token's `partials` rows of y) * w_post
    (w_post None: without the norm), then += emb[ids] (emb_add) or = emb[ids]; out = norm(resid) * w_next (w_next
    None: resid as it is). The norms are of `post_groups` and `next_groups` equal parts of a row. Depth average, with
    mix [n + 1]: resid joins hist (fp32 [n, T, D]) as its last entry, and becomes mix[0] emb[ids] + sum_j mix[j]
    hist[j - 1]. Returns out. `rows`: out row i is row rows[i]'s, and resid and hist keep their values."""
    if _on_gpu(resid):
        require_latent().residual_norm(resid, y, int(partials), float(y_scale), w_post, emb, ids, bool(emb_add),
                                       w_next, out, rows, float(eps), int(post_groups), int(next_groups), mix, hist)
        return out
    return ref.residual_norm(resid, eps, y, partials, y_scale, w_post, emb, ids, emb_add, w_next, out, rows, post_groups,
                             next_groups, mix, hist)


# ---- latent cache and attention ---------------------------------------------------------------
def latent_cache(x, nq: int, R: int, r: int, w_q, w_c, cq, pages, Rp: int, positions, slots, cos_sin, eps: float):
    """x [T, nq | R | r ...] -> cq = norm of the first nq columns, and the token's cache row: norm of the
    next R, and the rotated last r (csrc/ops/latent_cache.hip). nq 0: no cq; r 0: no rotated part."""
    if _on_gpu(x):
        require_latent().latent_cache(x, int(nq), int(R), int(r), w_q, w_c, cq, pages, int(Rp), positions, slots,
                                      cos_sin, float(eps))
    else:
        ref.latent_cache(x, nq, R, r, w_q, w_c, cq, pages, Rp, positions, slots, cos_sin, eps)


def latent_attention(out, part_o, part_ml, q, pages, items, n_items, q_start, q_len, ctx_len, block_table,
                     scale: float, window: int, dec_tokens: int, tile_tokens: int, num_seqs: Optional[int] = None,
                     simple: bool = False):
    """Attention of absorbed queries q [T, H, D] over latent pages -> out [T, H, Rp]; `window` 0: none.
    dec_tokens / tile_tokens: the scheduler's items hold at most dec_tokens tokens (split over keys) or
    tile_tokens (csrc/ops/latent_attention.hip). `simple`: the any-size kernel."""
    if _on_gpu(q):
        require_latent().latent_attention(out, part_o, part_ml, q, pages, items, n_items, q_start, q_len,
                                          ctx_len, block_table, int(dec_tokens), int(tile_tokens), int(window),
                                          float(scale), bool(simple))
    else:
        ref.latent_attention(out, q, pages, q_start, q_len, ctx_len, block_table, scale, window,
                             len(q_len) if num_seqs is None else num_seqs)
    return out


# ---- grouped projections ----------------------------------------------------------------------
def pack_groups(w: torch.Tensor, dtype) -> torch.Tensor:
    """[G, N, K] (N % 16 == 0, K % 32 == 0) -> the layout grouped_gemm.hip reads: MFMA fragments in bf16
    ([G, N/16, K/32, 64, 8]), row-major in fp32."""
    G, N, K = w.shape
    w = w.to(dtype)
    if dtype == torch.float32:
        return w.contiguous()
    return w.reshape(G, N // 16, 16, K // 32, 4, 8).permute(0, 1, 3, 4, 2, 5).reshape(G, N // 16, K // 32, 64, 8) \
        .contiguous()


def unpack_groups(wp: torch.Tensor) -> torch.Tensor:
    if wp.dim() == 3:
        return wp
    G, A, S = wp.shape[:3]
    return wp.view(G, A, S, 4, 16, 8).permute(0, 1, 4, 2, 3, 5).reshape(G, A * 16, S * 32)


def interleave_gate_up(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
    """[G, F, K] x 2 (F % 16 == 0) -> [G, 2F, K], 16 gate rows before the 16 up rows of the same outputs."""
    G, F, K = gate.shape
    return torch.stack([gate.reshape(G, F // 16, 16, K), up.reshape(G, F // 16, 16, K)], 2).reshape(G, 2 * F, K)


def head_gemm(x, x_step: int, w, out, out_step: int, rot: Optional[tuple] = None, gate: Optional[torch.Tensor] = None):
    """out[:, g * out_step : + N] = x[:, g * x_step : + K] @ w[g].T for every group g, times sigmoid(gate) (columns as
    out's) if given. rot = (positions, cos_sin, skip, r, rp): beside them, out[:, g * out_step + N : + rp] = x[:, g *
    x_step + skip : + r] rotated by the row's position and padded with zeros."""
    if _on_gpu(x):
        pos, cs, skip, r, rp = rot or (None, None, 0, 0, 0)
        require_grouped().head_gemm(x, int(x_step), w, out, int(out_step), pos, cs, int(skip), int(r), int(rp), gate)
    else:
        ref.head_gemm(x, x_step, unpack_groups(w), out, out_step, rot, gate)
    return out


def table_gemm(x, w, out, table, ids, col: int, glu: tuple):
    """out[:, :N] = the gated unit (limit, alpha, bias[, cubic]) of x @ w.T and table[ids, col : col + N]."""
    lim, alpha, bias, cubic = (tuple(glu) + (0.0,))[:4]
    if _on_gpu(x):
        require_grouped().table_gemm(x, w, out, table, ids, int(col), float(lim), float(alpha), float(bias), float(cubic))
    else:
        ref.table_gemm(x, unpack_groups(w)[0], out, table, ids, col, lim, alpha, bias, cubic)
    return out


def table_route(tables, desc, desc_host, ids, slots, T: int, tm: int, order, tiles, n_tiles):
    """Sort every layer's (token, choice) pairs by expert, from the layers' token tables, in one launch
    (grouped_gemm.hip table_route_kernel)."""
    if _on_gpu(ids):
        require_family("latent").table_route(tables, desc, desc_host, ids, slots, int(T), int(tm), order, tiles, n_tiles)
    else:
        ref.table_route(tables, desc_host, ids, slots, T, tm, order, tiles, n_tiles)


def expert_gemm(x, w, out, tiles, n_tiles, order, rows: int, *, x_div: int, out_order: bool, tm: int,
                glu: Optional[tuple] = None, relu2: bool = False, row_w: Optional[torch.Tensor] = None):
    """Rows sorted by expert: out row = x row @ w[expert].T; glu = (limit, alpha, bias[, cubic]): the gated
    pair of interleave_gate_up weights, min(g, limit) sigmoid(alpha (g + cubic g^3)) (clamp(u) + bias); relu2: the
    square of what is positive. x row = order[p] // x_div (0: p), out row = order[p] if out_order. row_w (with glu
    and x_div): x's row is multiplied by row_w[order[p]]."""
    lim, alpha, bias, cubic = (tuple(glu) + (0.0,))[:4] if glu else (0.0, 0.0, 0.0, 0.0)
    if _on_gpu(x):
        require_grouped().expert_gemm(x, w, out, tiles, n_tiles, order, int(rows), int(x_div), bool(out_order), int(tm),
                                      1 if glu is not None else 2 if relu2 else 0, float(lim), float(alpha), float(bias), float(cubic),
                                      row_w)
    else:
        ref.expert_gemm(x, unpack_groups(w), out, tiles, n_tiles, order, x_div, out_order, glu, relu2, row_w)
    return out


# ---- gated linear attention -------------------------------------------------------------------
def linear_attention(x, y, state, a2, bias, q_start, q_len, ctx_len, state_slot, scan_items, n_scan, cols, q_scale: float,
                     inv_tau: float, scan_min: int = SCAN_MIN, num_seqs: Optional[int] = None):
    """The recurrence S <- diag(e^g) S + k v^T, y = S^T q q_scale over the step's portions, from and to the sequences'
    state slots, with g = logsigmoid(a2 a + bias) inv_tau for every key channel (csrc/ops/linear_attention.hip). cols:
    columns of x where q, k, v and the low-rank inputs a start. state fp32 [slots, H, V, N], a2 [H N, rank]."""
    H, V, N = state.shape[1:]
    if not _on_gpu(x):
        ref.linear_attention(x, y, state, a2, bias, q_start, q_len, ctx_len, state_slot, cols, q_scale, inv_tau,
                             len(q_len) if num_seqs is None else num_seqs)
        return y
    T = x.shape[0]
    seqs = min(T, q_len.numel())
    items = 0 if T <= scan_min else min(scan_items.shape[0], T // SCAN_CHUNK + min(seqs, T // (scan_min + 1)) + 1)
    chunked = items if x.dtype == torch.bfloat16 else 0
    new = lambda dt, *s: torch.empty(*s, dtype=dt, device=x.device)  # noqa: E731
    rows = T if chunked else 0
    qd, kd, sc = (new(x.dtype, 2, rows, H, n) for n in (N, N, SCAN_CHUNK))
    require_family("latent_linear").linear_attention(
        x, y, state, new(torch.float32, chunked, H, V, N), qd, kd, sc, new(torch.float32, chunked, H, N), a2, bias, q_start, q_len,
        ctx_len, state_slot, scan_items, n_scan, int(chunked), int(seqs), [int(c) for c in cols], float(q_scale), float(inv_tau),
        int(scan_min))
    return y


# ---- activations ------------------------------------------------------------------------------
def poly_norm(z, n: int, act, eps: float):
    """z[:, :n] = a z / rms(z) + b z^2 / rms(z^2) + c z^3 / rms(z^3) + e with act = (a, b, c, e), in place; z's other
    columns are cleared (csrc/ops/poly_norm.hip)."""
    if _on_gpu(z):
        require_family("latent_linear").poly_norm(z, int(n), act, float(eps))
    else:
        ref.poly_norm(z, n, act, eps)
    return z
