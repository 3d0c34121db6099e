"""Dispatch of the fp32-residual, latent-attention and grouped-projection kernels (module _latent).

Device tensors run the HIP kernels of csrc/ops/{residual_norm, latent_cache, latent_attention,
grouped_gemm}.hip and raise when the module is missing; CPU tensors run the fp32 references of
ops/reference.py. Every function takes its constants as arguments and works in bf16 or fp32.
"""
from __future__ import annotations

from typing import Optional

import torch

from . import reference as ref
from .kernels import _on_gpu, require_grouped, require_latent

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
                  out: Optional[torch.Tensor] = None, rows: Optional[torch.Tensor] = None):
    """resid (fp32 [T, D], in place) += norm(y_scale * sum of a token's `partials` rows of y) * w_post
    (w_post None: without the norm), then += emb[ids] (emb_add) or = emb[ids]; out = norm(resid) * w_next.
    Returns out. `rows`: out row i is row rows[i]'s, and resid keeps its value."""
    if _on_gpu(resid):
        require_latent().residual_norm(resid, y, int(partials), float(y_scale), w_post, emb, ids, bool(emb_add),
                                       w_next, out, rows, float(eps))
        return out
    return ref.residual_norm(resid, eps, y, partials, y_scale, w_post, emb, ids, emb_add, w_next, out, rows)


# ---- latent cache and attention ---------------------------------------------------------------
def latent_cache(x, nq: int, R: int, r: int, w_q, w_c, cq, pages, Rp: int, positions, slots, cos_sin, eps: float):
    """x [T, nq | R | r ...] -> cq = norm of the first nq columns, and the token's cache row: norm of the
    next R, and the rotated last r (csrc/ops/latent_cache.hip)."""
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


def head_gemm(x, x_step: int, w, out, out_step: int, rot: Optional[tuple] = None):
    """out[:, g * out_step : + N] = x[:, g * x_step : + K] @ w[g].T for every group g. rot = (positions,
    cos_sin, skip, r, rp): beside them, out[:, g * out_step + N : + rp] = x[:, g * x_step + skip : + r] rotated
    by the row's position and padded with zeros."""
    if _on_gpu(x):
        pos, cs, skip, r, rp = rot or (None, None, 0, 0, 0)
        require_grouped().head_gemm(x, int(x_step), w, out, int(out_step), pos, cs, int(skip), int(r), int(rp))
    else:
        ref.head_gemm(x, x_step, unpack_groups(w), out, out_step, rot)
    return out


def table_route(tables, desc, desc_host, ids, slots, T: int, tm: int, order, tiles, n_tiles):
    """Sort every layer's (token, choice) pairs by expert, from the layers' token tables, in one launch
    (grouped_gemm.hip table_route_kernel)."""
    if _on_gpu(ids):
        require_latent().table_route(tables, desc, desc_host, ids, slots, int(T), int(tm), order, tiles, n_tiles)
    else:
        ref.table_route(tables, desc_host, ids, slots, T, tm, order, tiles, n_tiles)


def expert_gemm(x, w, out, tiles, n_tiles, order, rows: int, *, x_div: int, out_order: bool, tm: int,
                glu: Optional[tuple] = None, relu2: bool = False):
    """Rows sorted by expert: out row = x row @ w[expert].T; glu = (limit, alpha, bias[, cubic]): the gated
    pair of interleave_gate_up weights, min(g, limit) sigmoid(alpha (g + cubic g^3)) (clamp(u) + bias); relu2: the
    square of what is positive. x row = order[p] // x_div (0: p), out row = order[p] if out_order."""
    lim, alpha, bias, cubic = (tuple(glu) + (0.0,))[:4] if glu else (0.0, 0.0, 0.0, 0.0)
    if _on_gpu(x):
        require_grouped().expert_gemm(x, w, out, tiles, n_tiles, order, int(rows), int(x_div), bool(out_order), int(tm),
                                      1 if glu is not None else 2 if relu2 else 0, float(lim), float(alpha), float(bias), float(cubic))
    else:
        ref.expert_gemm(x, unpack_groups(w), out, tiles, n_tiles, order, x_div, out_order, glu, relu2)
    return out
