"""Dispatch of the hybrid models' kernels (module _hybrid): attention over paged keys and values with its
masks, biases and gates, state-space and matrix-memory layers, score-routed experts and fp32 residuals.

Device tensors run the HIP kernels of csrc/ops/{hyper_norm, paged_kv, window_attention, head_difference,
state_scan, matrix_memory, gated_norm, score_route}.hip and raise when the module is missing; CPU tensors run the fp32 references of
ops/reference.py. Every function takes its constants as arguments and works in bf16 or fp32.
"""
from __future__ import annotations

from typing import Optional

import torch

from . import reference as ref
from .kernels import MIXED, _on_gpu, require_family, require_hybrid
from .latent import SCAN_CHUNK, SCAN_MIN, unpack_groups

# (key width, value width) in 32s with MFMA kernels (window_attention.hip PA_WA_DIMS)
WINDOW_TILES = ((1, 1), (1, 2), (2, 1), (2, 2), (2, 4), (3, 3), (4, 2), (4, 4), (4, 8), (6, 4), (6, 6), (8, 8))
CONV_TAPS = (4, 8)  # built convolutions: shorter ones get zero taps in front


def window_pad(k: int, v: int) -> tuple:
    """Cached key and value widths: the first pair with an MFMA kernel that holds both, else whole 32s."""
    a, b = (k + 31) // 32, (v + 31) // 32
    a, b = next(((x, y) for x, y in WINDOW_TILES if a <= x and b <= y), (a, b))
    return 32 * a, 32 * b


def pooled_per_page(pool: int) -> int:
    """Blocks of `pool` tokens that can end in one page of 16."""
    return max(1, (16 + pool - 1) // pool) if pool > 0 else 1


def conv_taps(taps: int) -> int:
    return next(t for t in CONV_TAPS if taps <= t)


# ---- residual -----------------------------------------------------------------------------------
def hyper_norm(x: torch.Tensor, eps: float, *, y: Optional[torch.Tensor] = None, partials: int = 1,
               y_weights: Optional[torch.Tensor] = None, y2: Optional[torch.Tensor] = None,
               bias: Optional[torch.Tensor] = None, mix: Optional[torch.Tensor] = None, post: Optional[torch.Tensor] = None,
               pre: Optional[torch.Tensor] = None, emb: Optional[torch.Tensor] = None,
               ids: Optional[torch.Tensor] = None, w_next: Optional[torch.Tensor] = None,
               out: Optional[torch.Tensor] = None, rows: Optional[torch.Tensor] = None):
    """x (fp32 [T, streams, D], in place): x_t = sum_s mix[s, t] x_s + post[t] (sum_k w_k y_k + y2 + bias), or
    x_t = emb[ids]; out = norm(sum_s pre[s] x_s) * w_next. Returns out. `rows`: out row i is row rows[i]'s,
    and x keeps its value."""
    if _on_gpu(x):
        require_hybrid().hyper_norm(x, y, int(partials), y_weights, y2, bias, mix, post, pre, emb, ids, w_next, out, rows,
                                    float(eps))
        return out
    return ref.hyper_norm(x, eps, y, partials, y_weights, y2, bias, mix, post, pre, emb, ids, w_next, out, rows)


def softcap(x: torch.Tensor, cols: int, cap: float) -> torch.Tensor:
    """x[:, :cols] = cap * tanh(x / cap), in place."""
    if _on_gpu(x):
        require_hybrid().softcap(x, int(cols), float(cap))
    else:
        x[:, :cols] = (cap * torch.tanh(x[:, :cols].float() / cap)).to(x.dtype)
    return x


# ---- attention ----------------------------------------------------------------------------------
def paged_kv(x, bias, q, kp, vp, pk, pv, positions, slots, q_start, q_len, ctx_len, block_table, cos_sin, pool: int,
             num_seqs: Optional[int] = None, *, v_col: int = -1, q_norm: Optional[torch.Tensor] = None,
             k_norm: Optional[torch.Tensor] = None, norm_v: bool = False, dim: int = 0, vdim: int = 0, eps: float = 0.0):
    """Projection rows [q heads | k heads | v heads] -> queries q [T, H, DK], paged keys and values, and the mean
    rows of the blocks of `pool` tokens that end here (csrc/ops/paged_kv.hip). v_col: the values' first column,
    if not behind the keys. q_norm, k_norm [DK]: every query and key head normed over its `dim` real values;
    norm_v: value heads likewise over `vdim`, without a weight. Then the rotation (cos_sin None: none)."""
    if _on_gpu(x):
        require_hybrid().paged_kv(x, bias, q, kp, vp, pk, pv, positions, slots, q_start, q_len, ctx_len, block_table,
                                  cos_sin, int(pool), int(v_col), q_norm, k_norm, bool(norm_v), int(dim), int(vdim),
                                  float(eps))
    else:
        ref.paged_kv(x, bias, q, kp, vp, pk, pv, positions, slots, q_start, q_len, ctx_len, block_table, cos_sin, pool,
                     v_col, q_norm, k_norm, norm_v, dim, vdim, eps, len(q_len) if num_seqs is None else num_seqs)


def window_attention(out, part_o, part_ml, q, kp, vp, pk, pv, items, n_items, q_start, q_len, ctx_len, block_table,
                     scale: float, window: int, pool: int, sink: Optional[torch.Tensor], dec_tokens: int,
                     tile_tokens: int, max_slots: int, num_seqs: Optional[int] = None, simple: bool = False, *,
                     keep: int = 0, chunk: int = 0, slopes: Optional[torch.Tensor] = None, cap: float = 0.0,
                     gate: Optional[torch.Tensor] = None, gain: float = 1.0):
    """Grouped-query attention over pages: keys 0 <= i - j < window (0: all before i) and the first `keep`, of i's
    chunk of `chunk` positions (0: no chunks); the mean rows of whole blocks of `pool` tokens before the window (0:
    none). Scores q . k scale, capped (cap tanh(s / cap)) if cap > 0, less slopes[h] (i - j); exp(sink[h]) joins the
    softmax's denominator. out = gain * o * sigmoid(gate) in out's dtype; several key heads may share a value head.
    dec_tokens / tile_tokens: what the scheduler's items hold at most; max_slots: partial-result slots
    (csrc/ops/window_attention.hip). `simple`: the any-size kernel."""
    if _on_gpu(q):
        require_hybrid().window_attention(out, part_o, part_ml, q, kp, vp, pk, pv, items, n_items, q_start, q_len,
                                          ctx_len, block_table, int(dec_tokens), int(tile_tokens), int(window),
                                          int(pool), int(keep), int(chunk), float(scale), slopes, float(cap), sink, gate,
                                          float(gain), int(max_slots), bool(simple))
    else:
        ref.window_attention(out, q, kp, vp, pk, pv, q_start, q_len, ctx_len, block_table, scale, window, pool, keep,
                             chunk, slopes, cap, sink, gate, gain, len(q_len) if num_seqs is None else num_seqs)
    return out


def head_difference(a, out, gate, groups: int, lam: float, gain: float, vdim: int, eps: float):
    """Differential attention's second half: a fp32 [T, 2 H, D], heads (KV head, map, query head) -> out [T, H, D] =
    gain * norm(a_1 - lam a_2) * sigmoid(gate), normed over vdim real values (csrc/ops/head_difference.hip)."""
    if _on_gpu(a):
        require_hybrid().head_difference(a, out, gate, int(groups), float(lam), float(gain), int(vdim), float(eps))
    else:
        ref.head_difference(a, out, gate, groups, lam, gain, vdim, eps)
    return out


# ---- recurrent layers ---------------------------------------------------------------------------
def state_scan(proj, y, state, ring, conv_w, conv_b, dt_bias, a, d, q_start, q_len, ctx_len, state_slot, scan_first,
               scan_items, n_scan, groups: int, scan_min: int = SCAN_MIN, num_seqs: Optional[int] = None):
    """Convolution, silu and the recurrence S <- exp(-a dt) S + dt B x^T, y = S^T C + d x over the step's
    portions, from and to the sequences' state slots (csrc/ops/state_scan.hip). proj rows [z | x | B | C | dt]."""
    H, V, N = state.shape[1:]
    if not _on_gpu(proj):
        ref.state_scan(proj, y, state, ring, conv_w, conv_b, dt_bias, a, d, q_start, q_len, ctx_len, state_slot, groups,
                       len(q_len) if num_seqs is None else num_seqs)
        return y
    T = proj.shape[0]
    seqs = min(T, q_len.numel())
    items = 0 if T <= scan_min else min(scan_items.shape[0], T // SCAN_CHUNK + min(seqs, T // (scan_min + 1)) + 1)
    new = lambda dt, *s: torch.empty(*s, dtype=dt, device=proj.device)  # noqa: E731
    u = new(proj.dtype, T if items else 0, ring.shape[2])
    chunked = items if proj.dtype == torch.bfloat16 else 0
    work, total = new(torch.float32, chunked, H, V, N), new(torch.float32, chunked, H)
    require_hybrid().state_scan(proj, u, y, state, ring, work, total, conv_w, conv_b, dt_bias, a, d, q_start, q_len, ctx_len,
                                state_slot, scan_first, scan_items, n_scan, int(items), int(seqs), int(groups),
                                int(scan_min))
    return y


def matrix_memory(x, y, div, state, top, i_bias, f_bias, q_start, q_len, ctx_len, state_slot, scan_items, n_scan, cols,
                  vdim: int, cap: float, q_scale: float, scan_min: int = SCAN_MIN, num_seqs: Optional[int] = None):
    """The recurrence m' = max(f + m, i), S' = e^(f + m - m') S + e^(i - m') v k^T over the step's portions, from and
    to the sequences' state slots: y = S' q q_scale [T, H * vin] and div [T, H] = max(|n . q|, e^-m') + 1e-6, where
    n, the sum of the keys, is S's row `vdim` (csrc/ops/matrix_memory.hip). cols: columns of x where q, k, v and the
    gates i | f start, and a value head's width vin. state fp32 [slots, H, V, N], top (m) fp32 [slots, H, V]."""
    H, V, N = state.shape[1:]
    if not _on_gpu(x):
        ref.matrix_memory(x, y, div, state, top, i_bias, f_bias, q_start, q_len, ctx_len, state_slot, cols, vdim, cap, q_scale,
                          len(q_len) if num_seqs is None else num_seqs)
        return y
    T = x.shape[0]
    seqs = min(T, q_len.numel())
    items = 0 if T <= scan_min else min(scan_items.shape[0], T // SCAN_CHUNK + min(seqs, T // (scan_min + 1)) + 1)
    chunked = items if x.dtype == torch.bfloat16 else 0
    work = torch.empty(chunked, H, V, N, dtype=torch.float32, device=x.device)
    stat = torch.empty(chunked, H, 4, dtype=torch.float32, device=x.device)
    require_hybrid().matrix_memory(x, y, div, state, top, work, stat, i_bias, f_bias, q_start, q_len, ctx_len, state_slot,
                                   scan_items, n_scan, int(chunked), int(seqs), [int(c) for c in cols], int(vdim), float(cap),
                                   float(q_scale), int(scan_min))
    return y


def gated_norm(y, z, w, slots, heads: int, vdim: int, vpad: int, parts: int, eps: float,
               div: Optional[torch.Tensor] = None, after: Optional[str] = None):
    """y (in place) = norm(y * silu(z)) * w, or with `after` ("sigmoid", "silu") norm(y) * w * after(z), normed in `parts`
    equal parts of the heads * vdim real columns; column h * vpad + v holds head h's v. div [T, heads]: y is divided by it
    first (csrc/ops/gated_norm.hip)."""
    if _on_gpu(y):
        require_family(*MIXED).gated_norm(y, z, w, slots, int(heads), int(vdim), int(vpad), int(parts), float(eps), div,
                                          (None, "sigmoid", "silu").index(after))
    else:
        ref.gated_norm(y, z, w, heads, vdim, vpad, parts, eps, div, after)
    return y


# ---- routing ------------------------------------------------------------------------------------
def score_route(h, w, slots, weights, choice, rank, counts, order, tiles, n_tiles, E: int, top: int, groups: int,
                keep: int, always: int, tm: int, *, softmax: bool = False, correction: Optional[torch.Tensor] = None,
                share: bool = False, scale: float = 1.0):
    """Choose each token's `top` of E experts by s = sigmoid(w h) (or softmax(w h)) + correction, limited to the `keep`
    best of `groups` groups (scored by their two best members), with weights scale * s (`share`: s / (sum of the
    chosen s + 1e-20)); `always` more experts follow with weight 1. Writes weights [T, top + always] and the rows
    sorted by expert (csrc/ops/score_route.hip). counts: E + always zeros when there are more than 16 rows."""
    if _on_gpu(h):
        require_family(*MIXED).score_route(h, w, slots, weights, choice, rank, counts, order, tiles, n_tiles, int(E), int(top),
                                     int(groups), int(keep), int(always), int(tm), bool(softmax), correction, bool(share),
                                     float(scale))
    else:
        ref.score_route(h, unpack_groups(w)[0], slots, weights, choice, order, tiles, n_tiles, E, top, groups, keep,
                        always, tm, softmax, correction, share, scale)
