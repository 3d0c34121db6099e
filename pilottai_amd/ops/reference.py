"""Plain-PyTorch fp32 reference implementations of every HIP kernel.

They define the semantics the CDNA4 kernels are tested against (GPU numerics
tests compare kernel output with these on the same inputs) and serve as the CPU
execution path for the control-plane tests that run without a GPU. On a GPU box
the native kernels are mandatory (see ops/kernels.py) — these are never a
silent fallback for device tensors.
"""
from __future__ import annotations

import math
from typing import Optional

import numpy as np
import torch

# ---------------------------------------------------------------------------
# normalisation / activation
# ---------------------------------------------------------------------------


def rmsnorm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    xf = x.float()
    inv = torch.rsqrt(xf.pow(2).mean(-1, keepdim=True) + eps)
    return ((xf * inv).to(x.dtype).float() * w.float()).to(x.dtype)


def fused_add_rmsnorm(resid: torch.Tensor, x: torch.Tensor, w: torch.Tensor, eps: float):
    """Returns (normed, new_resid); new_resid = bf16(resid + x)."""
    new_resid = (resid.float() + x.float()).to(resid.dtype)
    return rmsnorm(new_resid, w, eps), new_resid


def silu_mul(x: torch.Tensor) -> torch.Tensor:
    F = x.shape[-1] // 2
    g, u = x[..., :F].float(), x[..., F:].float()
    return (torch.nn.functional.silu(g).to(x.dtype).float() * u).to(x.dtype)


# ---------------------------------------------------------------------------
# RoPE + paged KV cache
# ---------------------------------------------------------------------------


def rope_cos_sin(max_pos: int, head_dim: int = 128, theta: float = 500000.0,
                 scaling: Optional[dict] = None) -> torch.Tensor:
    """fp32 [max_pos, head_dim] table: cos in [:, :hd/2], sin in [:, hd/2:].

    `scaling` follows the Llama-3.1 "llama3" rope_scaling dict (factor,
    low_freq_factor, high_freq_factor, original_max_position_embeddings).
    """
    half = head_dim // 2
    inv = 1.0 / (theta ** (torch.arange(0, half, dtype=torch.float64) / half))
    if scaling:
        factor = scaling.get("factor", 8.0)
        lo = scaling.get("low_freq_factor", 1.0)
        hi = scaling.get("high_freq_factor", 4.0)
        old = scaling.get("original_max_position_embeddings", 8192)
        lo_wl, hi_wl = old / lo, old / hi
        wl = 2 * math.pi / inv
        smooth = (old / wl - lo) / (hi - lo)
        scaled = torch.where(wl > lo_wl, inv / factor, inv)
        mid = (wl <= lo_wl) & (wl >= hi_wl)
        scaled = torch.where(mid, (1 - smooth) * inv / factor + smooth * inv, scaled)
        inv = scaled
    pos = torch.arange(max_pos, dtype=torch.float64)
    ang = torch.outer(pos, inv)
    return torch.cat([ang.cos(), ang.sin()], dim=1).float()


def apply_rope(x: torch.Tensor, positions: torch.Tensor, cos_sin: torch.Tensor) -> torch.Tensor:
    """x [T, heads, 128] -> rotated (bf16 rounding as in the kernel)."""
    half = x.shape[-1] // 2
    cs = cos_sin[positions.long()]
    c, s = cs[:, None, :half], cs[:, None, half:]
    x1, x2 = x[..., :half].float(), x[..., half:].float()
    o1 = x1 * c - x2 * s
    o2 = x2 * c + x1 * s
    return torch.cat([o1, o2], dim=-1).to(x.dtype)


def rope_cache(q_out, k_cache, v_cache, qkv, positions, slot_mapping, cos_sin, H, KV,
               apply: bool = True):
    T = qkv.shape[0]
    hd = 128
    q = qkv[:, : H * hd].reshape(T, H, hd)
    k = qkv[:, H * hd:(H + KV) * hd].reshape(T, KV, hd)
    v = qkv[:, (H + KV) * hd:(H + 2 * KV) * hd].reshape(T, KV, hd)
    if apply:
        q = apply_rope(q, positions[:T], cos_sin)
        k = apply_rope(k, positions[:T], cos_sin)
    q_out[:T].copy_(q.reshape(q_out[:T].shape))
    blk = k_cache.shape[3]  # K page: [KV, 128/8, block, 8] (fragment-major)
    for t in range(T):
        slot = int(slot_mapping[t])
        if slot < 0:
            continue
        b, o = divmod(slot, blk)
        k_cache[b, :, :, o, :] = k[t].reshape(KV, hd // 8, 8)
        v_cache[b, :, :, o] = v[t]


def paged_attention(q, k_cache, v_cache, q_start, q_len, ctx_len, block_table, scale):
    """q [T, H, 128]; returns out [T, H, 128] (fp32 math, causal within context)."""
    T, H, hd = q.shape
    KV = k_cache.shape[1]
    G = H // KV
    blk = k_cache.shape[3]
    out = torch.zeros_like(q)
    for s in range(len(q_len)):
        ql, ctx, q0 = int(q_len[s]), int(ctx_len[s]), int(q_start[s])
        if ql <= 0:
            continue
        nb = (ctx + blk - 1) // blk
        blocks = block_table[s, :nb].long()
        K = k_cache[blocks].permute(1, 0, 3, 2, 4).reshape(KV, nb * blk, hd)[:, :ctx].float()
        V = v_cache[blocks].permute(1, 0, 3, 2).reshape(KV, nb * blk, hd)[:, :ctx].float()
        Kh = K.repeat_interleave(G, dim=0)  # [H, ctx, hd]
        Vh = V.repeat_interleave(G, dim=0)
        qs = q[q0:q0 + ql].float().permute(1, 0, 2)  # [H, ql, hd]
        sc = torch.matmul(qs, Kh.transpose(1, 2)) * scale  # [H, ql, ctx]
        pos = torch.arange(ctx - ql, ctx)[:, None]
        keys = torch.arange(ctx)[None, :]
        sc = sc.masked_fill(keys > pos, float("-inf"))
        p = torch.softmax(sc, dim=-1)
        o = torch.matmul(p, Vh)  # [H, ql, hd]
        out[q0:q0 + ql] = o.permute(1, 0, 2).to(q.dtype)
    return out


# ---------------------------------------------------------------------------
# sampling — same counter-based hash as csrc/ops/common.h (uniform01)
# ---------------------------------------------------------------------------

_M32 = np.uint64(0xFFFFFFFF)


def _mix32(x: np.ndarray) -> np.ndarray:
    x = x.astype(np.uint64) & _M32
    x ^= x >> np.uint64(16)
    x = (x * np.uint64(0x7FEB352D)) & _M32
    x ^= x >> np.uint64(15)
    x = (x * np.uint64(0x846CA68B)) & _M32
    x ^= x >> np.uint64(16)
    return x


def uniform01(seed: int, row_off: int, cols: np.ndarray) -> np.ndarray:
    seed = int(seed) & 0xFFFFFFFFFFFFFFFF
    lo, hi = seed & 0xFFFFFFFF, seed >> 32
    a = _mix32(np.array([(row_off * 0x9E3779B9 + hi) & 0xFFFFFFFF], dtype=np.uint64))
    h = _mix32(np.uint64(lo) ^ a)
    c = (cols.astype(np.uint64) * np.uint64(0x85EBCA6B) + np.uint64(0x27D4EB2F)) & _M32
    h = _mix32(h ^ c)
    return ((h >> np.uint64(8)).astype(np.float64) + 0.5) * (1.0 / 16777216.0)


def topkp_threshold(logits: torch.Tensor, temperature, top_k, top_p, mask_class, class_masks):
    """Exact top-k / top-p logit threshold per row (fp64 math, sort based).

    Kept set = allowed tokens with logit >= tau; tau is the larger of the k-th
    largest allowed logit and the value at which the descending cumulative
    softmax(logit / T) mass first reaches p. -inf = no truncation."""
    rows, V = logits.shape
    out = torch.full((rows,), float("-inf"), dtype=torch.float32)
    lg = logits.float().cpu().numpy().astype(np.float64)
    cm = class_masks.cpu().numpy().view(np.uint32) if class_masks is not None else None
    for r in range(rows):
        T, k, p = float(temperature[r]), int(top_k[r]), float(top_p[r])
        if T <= 0 or ((k <= 0 or k >= V) and not p < 1.0):
            continue
        vals = lg[r]
        mc = int(mask_class[r])
        if mc >= 0 and cm is not None:
            idx = np.arange(V)
            ok = ((cm[mc][idx >> 5] >> (idx & 31).astype(np.uint32)) & 1).astype(bool)
            vals = vals[ok]
        if vals.size == 0:
            continue
        s = np.sort(vals)[::-1]
        t = -np.inf
        if 0 < k < s.size:
            t = max(t, s[k - 1])
        if p < 1.0:
            w = np.exp((s - s[0]) / T)
            c = np.cumsum(w)
            j = int(np.searchsorted(c, p * c[-1] * (1 - 1e-6)))
            t = max(t, s[min(j, s.size - 1)])
        out[r] = t
    return out


def sample(logits: torch.Tensor, temperature, mask_class, class_masks, seeds, offsets,
           forced=None, vocab_offset: int = 0, return_keys: bool = False, tau=None):
    """Gumbel-max sampling with grammar masks (and optional top-k/p threshold
    tau: logits below it are excluded); returns int32 tokens [rows]."""
    rows, V = logits.shape
    toks = torch.zeros(rows, dtype=torch.int32)
    keys_out = torch.zeros(rows, dtype=torch.float32)
    lg = logits.float().cpu().numpy().astype(np.float64)
    cm = class_masks.cpu().numpy().view(np.uint32) if class_masks is not None else None
    for r in range(rows):
        f = int(forced[r]) if forced is not None else -1
        T = float(temperature[r])
        mc = int(mask_class[r])
        idx = np.arange(V) + vocab_offset
        valid = np.ones(V, dtype=bool)
        if mc >= 0 and cm is not None:
            words = cm[mc][idx >> 5]
            valid = ((words >> (idx & 31).astype(np.uint32)) & 1).astype(bool)
        if T <= 0:
            key = lg[r].copy()
        else:
            key = lg[r] / T
            u = uniform01(int(seeds[r]), int(offsets[r]), idx)
            key = key + (-np.log(-np.log(u)))
        if tau is not None:
            valid &= lg[r] >= float(tau[r])
        key[~valid] = -np.inf
        best = int(np.argmax(key)) if valid.any() else 0
        keys_out[r] = float(key[best]) if valid.any() else float("-inf")
        toks[r] = f if f >= 0 else best + vocab_offset
    return (toks, keys_out) if return_keys else toks


# ---------------------------------------------------------------------------
# semantic index
# ---------------------------------------------------------------------------


def cosine_topk(queries, index, n_valid, K, row_priority, row_tags, row_expiry, q_min_priority,
                q_tags, now):
    """Returns (scores [Q,K] fp32, rows [Q,K] int32), rows -1 past the matches."""
    Q = queries.shape[0]
    sc = queries.float() @ index[:n_valid].float().T  # [Q, N]
    out_s = torch.full((Q, K), float("-inf"))
    out_r = torch.full((Q, K), -1, dtype=torch.int32)
    prio = row_priority[:n_valid].long()
    tags = row_tags[:n_valid].long()
    exp = row_expiry[:n_valid].float()
    alive = (exp == 0) | (exp > now)
    for q in range(Q):
        qt = int(q_tags[q])
        ok = (prio >= int(q_min_priority[q])) & ((tags & qt) == qt) & alive
        s = sc[q].masked_fill(~ok, float("-inf"))
        k = min(K, int(ok.sum()))
        if k == 0:
            continue
        v, i = torch.topk(s, k)
        out_s[q, :k] = v
        out_r[q, :k] = i.int()
    return out_s, out_r


def q16_topk(qv, qmeta, hi, lo, rmeta, n_valid, K, row_priority, row_tags, row_expiry, q_min_priority, q_tags,
             now):
    """Exact top-k over the 16-bit fixed-point index (csrc/ops/similarity_q16.hip semantics):
    score = float32(float64(v_q . v_r) * (float64(s_r) * float64(s_q))) with v = 256 hi + lo,
    the integer dot products exact in int64. qv [Q, 2, D] int8 (qh, ql), qmeta [Q, 2] (s_q, .),
    hi / lo fragment-major int8 tiles, rmeta [N, 2] (s_r, .)."""
    T, DS = hi.shape[0], hi.shape[1]
    unpack = lambda t: t.view(T, DS, 4, 16, 16).permute(0, 3, 1, 2, 4).reshape(T * 16, DS * 64)  # noqa: E731
    n = int(n_valid)
    vr = 256 * unpack(hi)[:n].long().cpu() + unpack(lo)[:n].long().cpu()
    vq = 256 * qv[:, 0].long().cpu() + qv[:, 1].long().cpu()
    dots = vq @ vr.T  # exact int64
    sc = (dots.double() * (rmeta[:n, 0].double().cpu()[None, :] * qmeta[:, 0].double().cpu()[:, None])).float()
    return cosine_topk_from_scores(sc, n, K, row_priority, row_tags, row_expiry, q_min_priority, q_tags, now)


def cosine_topk_from_scores(sc, n_valid, K, row_priority, row_tags, row_expiry, q_min_priority, q_tags, now):
    """The filtered top-k of precomputed scores [Q, n_valid] (the reference kernels' common tail)."""
    Q = sc.shape[0]
    out_s = torch.full((Q, K), float("-inf"))
    out_r = torch.full((Q, K), -1, dtype=torch.int32)
    prio = row_priority[:n_valid].long().cpu()
    tags = row_tags[:n_valid].long().cpu()
    exp = row_expiry[:n_valid].float().cpu()
    alive = (exp == 0) | (exp > now)
    for q in range(Q):
        qt = int(q_tags[q])
        ok = (prio >= int(q_min_priority[q])) & ((tags & qt) == qt) & alive
        s = sc[q].masked_fill(~ok, float("-inf"))
        k = min(K, int(ok.sum()))
        if k == 0:
            continue
        v, i = torch.topk(s, k)
        out_s[q, :k] = v
        out_r[q, :k] = i.int()
    return out_s, out_r


def pack_mask(allowed) -> torch.Tensor:
    """bool [V] -> int32 words, bit i of word i // 32 set iff token i is allowed."""
    a = np.asarray(allowed, dtype=bool)
    pad = (-len(a)) % 32
    if pad:
        a = np.concatenate([a, np.zeros(pad, dtype=bool)])
    return torch.from_numpy(np.packbits(a, bitorder="little").view(np.int32).copy())


# ---------------------------------------------------------------------------
# fp32 residual stream, latent attention, grouped projections (ops/latent.py)
# ---------------------------------------------------------------------------


def _norm32(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def _group_norm32(x: torch.Tensor, eps: float, groups: int) -> torch.Tensor:
    return _norm32(x.reshape(*x.shape[:-1], groups, -1), eps).reshape(x.shape)


def residual_norm(resid, eps, y, partials, y_scale, w_post, emb, ids, emb_add, w_next, out, rows, post_groups=1, next_groups=1,
                  mix=None, hist=None):
    T, D = resid.shape
    sel = torch.arange(T) if rows is None else rows.long()
    r = resid[sel]
    if y is not None:
        d = y[:, :D].float().view(T, partials, D).sum(1)[sel] * y_scale
        r = r + (_group_norm32(d, eps, post_groups) * w_post if w_post is not None else d)
    if emb is not None:
        e = emb[ids[:T].long()[sel].clamp(0, emb.shape[0] - 1)].float()
        if mix is not None:
            n = mix.numel() - 1
            if rows is None:
                hist[n - 1, :T] = r
            r = mix[0] * e + mix[n] * r + sum(mix[j] * hist[j - 1, :T][sel] for j in range(1, n))
        else:
            r = r + e if emb_add else e  # (set: before any y)
    if rows is None:
        resid.copy_(r)
    if out is not None:
        out[:len(sel), :D] = (_group_norm32(r, eps, next_groups) * w_next if w_next is not None else r).to(out.dtype)
        out[:len(sel), D:] = 0
    return out


def _rotate_part(x: torch.Tensor, positions: torch.Tensor, cos_sin: torch.Tensor) -> torch.Tensor:
    """fp32 [T, ..., r]: rotate-half over the first cos_sin.shape[1] of r dimensions."""
    rd = cos_sin.shape[1]
    half = rd // 2
    cs = cos_sin[positions.long()].view(x.shape[0], *([1] * (x.dim() - 2)), rd)
    c, s = cs[..., :half], cs[..., half:]
    u, v = x[..., :half], x[..., half:rd]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., rd:]], -1)


def latent_cache(x, nq, R, r, w_q, w_c, cq, pages, Rp, positions, slots, cos_sin, eps):
    T = x.shape[0]
    xf = x.float()
    if nq:
        cq.zero_()
        cq[:, :nq] = (_norm32(xf[:, :nq], eps) * w_q).to(cq.dtype)
    D = pages.shape[1] * 8
    row = torch.zeros(T, D)
    row[:, :R] = _norm32(xf[:, nq:nq + R], eps) * w_c
    if r:
        row[:, Rp:Rp + r] = _rotate_part(xf[:, nq + R:nq + R + r], positions[:T], cos_sin)
    for t in range(T):
        s = int(slots[t])
        if s >= 0:
            pages[s // 16, :, s % 16, :] = row[t].view(D // 8, 8).to(pages.dtype)


def latent_attention(out, q, pages, q_start, q_len, ctx_len, block_table, scale, window, num_seqs):
    Rp = out.shape[2]
    for s in range(num_seqs):
        n, ctx, q0 = int(q_len[s]), int(ctx_len[s]), int(q_start[s])
        if n <= 0:
            continue
        blk = block_table[s, :(ctx + 15) // 16].long()
        rows = pages[blk].permute(0, 2, 1, 3).reshape(-1, pages.shape[1] * 8)[:ctx].float()
        sc = torch.einsum("thd,kd->htk", q[q0:q0 + n].float(), rows) * scale
        back = torch.arange(ctx - n, ctx)[:, None] - torch.arange(ctx)[None, :]
        seen = (back >= 0) & (back < window) if window > 0 else back >= 0
        p = torch.softmax(sc.masked_fill(~seen, float("-inf")), -1)
        out[q0:q0 + n] = torch.einsum("htk,kd->thd", p, rows[:, :Rp]).to(out.dtype)


def head_gemm(x, x_step, w, out, out_step, rot, gate=None):
    N, K = w.shape[1:]
    for g in range(w.shape[0]):
        at = g * out_step
        y = x[:, g * x_step:g * x_step + K].float() @ w[g].float().T
        if gate is not None:
            y = y * torch.sigmoid(gate[:, at:at + N].float())
        out[:, at:at + N] = y.to(out.dtype)
        if rot is not None:
            pos, cs, skip, r, rp = rot
            out[:, at + N:at + N + rp] = 0
            v = x[:, g * x_step + skip:g * x_step + skip + r].float()
            out[:, at + N:at + N + r] = _rotate_part(v, pos[:x.shape[0]], cs).to(out.dtype)


def _gated_unit(g, u, lim, alpha, bias, cubic):
    g, u = g.clamp(max=lim), u.clamp(-lim, lim)
    return g * torch.sigmoid(alpha * (g + cubic * g ** 3)) * (u + bias)


def table_gemm(x, w, out, table, ids, col, lim, alpha, bias, cubic):
    N, K = w.shape
    e = table[ids[:x.shape[0]].long().clamp(0, table.shape[0] - 1), col:col + N].float()
    out[:, :N] = _gated_unit(x[:, :K].float() @ w.float().T, e, lim, alpha, bias, cubic).to(out.dtype)


def table_route(tables, desc, ids, slots, T, tm, order, tiles, n_tiles):
    for layer in range(desc.shape[0]):
        off, V, top, E, o0, t0, tmax, _ = (int(v) for v in desc[layer])
        tab = tables[off:off + V * top].view(V, top)
        e = tab[ids[:T].long().clamp(0, V - 1)].clamp(0, E - 1).reshape(-1)
        live = (slots[:T] >= 0).repeat_interleave(top)
        p = torch.arange(T * top)[live]
        p = p[torch.argsort(e[p], stable=True)]
        order[o0:o0 + len(p)] = p.to(torch.int32)
        k, start = 0, 0
        for x, c in enumerate(torch.bincount(e[p].long(), minlength=E).tolist()):
            for i in range(0, c, tm):
                tiles[t0 + k] = torch.tensor([x, start + i, min(tm, c - i), 0], dtype=torch.int32)
                k += 1
            start += c
        n_tiles[layer] = min(k, tmax)


def expert_gemm(x, w, out, tiles, n_tiles, order, x_div, out_order, glu, relu2=False, row_w=None):
    K = w.shape[2]
    for e, start, n, _ in tiles[:int(n_tiles[0])].tolist():
        p = torch.arange(start, start + n)
        xr = order[p].long() // x_div if x_div else p
        y = x[xr, :K].float() @ w[e].float().T
        if row_w is not None:
            y = y * row_w.reshape(-1)[order[p].long()][:, None]
        if glu is not None:
            y = y.view(n, -1, 2, 16)
            y = _gated_unit(y[:, :, 0].reshape(n, -1), y[:, :, 1].reshape(n, -1), *(tuple(glu) + (0.0,))[:4])
        if relu2:
            y = y.clamp(min=0) ** 2
        out[order[p].long() if out_order else p, :y.shape[1]] = y.to(out.dtype)


# ---------------------------------------------------------------------------
# residual of several streams, paged attention, recurrent layers, score routing (ops/hybrid.py)
# ---------------------------------------------------------------------------


def yarn_frequencies(dims: int, base: float, factor: float, original: float, fast: float, slow: float):
    """Angles per position of dims / 2 pairs: pairs that turn often within `original` positions keep theirs,
    slow ones are divided by `factor`, a linear ramp lies between; and the factor of cos and sin."""
    f = base ** (-2.0 * torch.arange(dims // 2, dtype=torch.float64) / dims)
    at = lambda turns: dims * math.log(original / (2 * math.pi * turns)) / (2 * math.log(base))  # noqa: E731
    lo, hi = max(math.floor(at(fast)), 0), min(math.ceil(at(slow)), dims - 1)
    ramp = ((torch.arange(dims // 2, dtype=torch.float64) - lo) / max(hi - lo, 0.001)).clamp(0, 1)
    return f * (1 - ramp) + f / factor * ramp, 0.1 * math.log(factor) + 1


def slow_wave_frequencies(dims: int, base: float, factor: float, low: float, high: float, original: float):
    """Angles per position of dims / 2 pairs, scaled by wavelength as in Llama 3.1: pairs that turn more than
    `high` times within `original` positions keep theirs, those that turn less than `low` times are divided by
    `factor`, and in between the two are mixed."""
    f = base ** (-2.0 * torch.arange(dims // 2, dtype=torch.float64) / dims)
    turns = original * f / (2 * math.pi)
    keep = ((turns - low) / (high - low)).clamp(0, 1) if high > low else (turns >= low).double()
    return f * keep + f / factor * (1 - keep)


def angle_table(max_pos: int, dims: int, base: float, yarn: Optional[dict] = None,
                slow_waves: Optional[dict] = None) -> torch.Tensor:
    """fp32 [max_pos, dims]: cos | sin of the rotate-half pairs, scaled if `yarn` (factor, original, fast, slow)
    or `slow_waves` (factor, low, high, original) is given."""
    if yarn:
        f, m = yarn_frequencies(dims, base, **yarn)
    elif slow_waves:
        f, m = slow_wave_frequencies(dims, base, **slow_waves), 1.0
    else:
        f, m = base ** (-2.0 * torch.arange(dims // 2, dtype=torch.float64) / dims), 1.0
    a = torch.arange(max_pos, dtype=torch.float64)[:, None] * f[None, :]
    return torch.cat([a.cos() * m, a.sin() * m], 1).float()


def hyper_norm(x, eps, y, partials, y_weights, y2, bias, mix, post, pre, emb, ids, w_next, out, rows):
    T, S, D = x.shape
    sel = torch.arange(T) if rows is None else rows.long()
    r = x[sel]
    if emb is not None:
        r = emb[ids[:T].long()[sel].clamp(0, emb.shape[0] - 1)].float()[:, None].expand(-1, S, -1)
    if y is not None:
        v = y[:, :D].float().view(T, partials, D)[sel]
        v = (v * y_weights.view(T, partials)[sel][:, :, None]).sum(1) if y_weights is not None else v.sum(1)
        if y2 is not None:
            v = v + y2[:, :D].float()[sel]
        if bias is not None:
            v = v + bias
        r = torch.einsum("st,nsd->ntd", mix, r) + post[None, :, None] * v[:, None]
    if rows is None:
        x.copy_(r)
    if out is not None:
        u = (pre[None, :, None] * r).sum(1)
        out[:len(sel), :D] = (_norm32(u, eps) * w_next).to(out.dtype)
        out[:len(sel), D:] = 0
    return out


def _page_rows(pages, blocks, n):
    """[n, G, D] fp32: a sequence's first n cached rows."""
    NB, G, d8 = pages.shape[:3]
    return pages[blocks.long()].permute(0, 3, 1, 2, 4).reshape(-1, G, d8 * 8)[:n].float()


def paged_kv(x, bias, q, kp, vp, pk, pv, positions, slots, q_start, q_len, ctx_len, block_table, cos_sin, pool, v_col,
             q_norm, k_norm, norm_v, dim, vdim, eps, num_seqs):
    T, H, DK = q.shape
    G, GV, DV = kp.shape[1], vp.shape[1], vp.shape[2] * 8
    at = (H + G) * DK if v_col < 0 else v_col
    r = x[:, :max((H + G) * DK, at + GV * DV)].float()
    if bias is not None:
        r = r + bias
    heads = r[:, :(H + G) * DK].view(T, H + G, DK)
    mean_norm = lambda h, n: h * torch.rsqrt(h.pow(2).sum(-1, keepdim=True) / n + eps)  # noqa: E731
    if q_norm is not None:
        w = torch.cat([q_norm.expand(H, -1), k_norm.expand(G, -1)])
        heads = mean_norm(heads, dim) * w
    if cos_sin is not None:
        heads = _rotate_part(heads, positions[:T], cos_sin)
    q.copy_(heads[:, :H].to(q.dtype))
    k, v = heads[:, H:], r[:, at:at + GV * DV].view(T, GV, DV)
    if norm_v:
        v = mean_norm(v, vdim)
    for t in range(T):
        s = int(slots[t])
        if s >= 0:
            kp[s // 16, :, :, s % 16] = k[t].view(G, -1, 8).to(kp.dtype)
            vp[s // 16, :, :, s % 16] = v[t].view(GV, -1, 8).to(vp.dtype)
    if pool <= 0:
        return
    for s in range(num_seqs):
        ctx, n = int(ctx_len[s]), int(q_len[s])
        if n <= 0:
            continue
        blocks = block_table[s, :(ctx + 15) // 16]
        kr, vr = _page_rows(kp, blocks, ctx), _page_rows(vp, blocks, ctx)
        for b in range((ctx - n) // pool, ctx // pool):
            page = (b * pool + pool - 1) // 16
            sub = b - page * 16 // pool
            pk[int(blocks[page]), sub] = kr[b * pool:(b + 1) * pool].mean(0).to(pk.dtype)
            pv[int(blocks[page]), sub] = vr[b * pool:(b + 1) * pool].mean(0).to(pv.dtype)


def window_attention(out, q, kp, vp, pk, pv, q_start, q_len, ctx_len, block_table, scale, window, pool, keep, chunk,
                     slopes, cap, sink, gate, gain, num_seqs):
    H, G, GV = q.shape[1], kp.shape[1], vp.shape[1]
    for s in range(num_seqs):
        n, ctx, q0 = int(q_len[s]), int(ctx_len[s]), int(q_start[s])
        if n <= 0:
            continue
        blocks = block_table[s, :(ctx + 15) // 16]
        k, v = _page_rows(kp, blocks, ctx), _page_rows(vp, blocks, ctx)
        pos, key = torch.arange(ctx - n, ctx)[:, None], torch.arange(ctx)[None, :]
        back = pos - key
        seen = (back >= 0) & ((back < window) | (key < keep)) if window > 0 else back >= 0
        if chunk > 0:
            seen = seen & (pos // chunk == key // chunk)
        if pool > 0 and window > 0 and ctx // pool:
            ends = torch.arange(ctx // pool) * pool + pool - 1
            page = blocks[ends // 16].long()
            sub = torch.arange(ctx // pool) - ends // 16 * 16 // pool
            k, v = torch.cat([k, pk[page, sub].float()]), torch.cat([v, pv[page, sub].float()])
            seen = torch.cat([seen, ends[None, :] <= pos - window], 1)
        k, v = k.repeat_interleave(H // G, 1), v.repeat_interleave(H // GV, 1)
        sc = torch.einsum("thd,khd->htk", q[q0:q0 + n].float(), k) * scale
        if cap > 0:
            sc = cap * torch.tanh(sc / cap)
        if slopes is not None:
            sc = sc - slopes[:, None, None] * back.float()
        sc = sc.masked_fill(~seen, float("-inf"))
        m = sc.amax(-1, keepdim=True)
        if sink is not None:
            m = torch.maximum(m, sink[:, None, None])
        p = torch.exp(sc - m)
        p = p / (p.sum(-1, keepdim=True) + (torch.exp(sink[:, None, None] - m) if sink is not None else 0))
        o = torch.einsum("htk,khd->thd", p, v) * gain
        if gate is not None:
            o = o * torch.sigmoid(gate[q0:q0 + n].float().view(o.shape))
        out[q0:q0 + n] = o.to(out.dtype)


def head_difference(a, out, gate, groups, lam, gain, vdim, eps):
    T, H2, D = a.shape
    m = a.float().view(T, groups, 2, H2 // (2 * groups), D)
    o = (m[:, :, 0] - lam * m[:, :, 1]).reshape(T, H2 // 2, D)
    o = o * torch.rsqrt(o.pow(2).sum(-1, keepdim=True) / vdim + eps) * gain
    out[:, :, :] = (o * torch.sigmoid(gate.float().view(o.shape))).to(out.dtype)


def state_scan(proj, y, state, ring, conv_w, conv_b, dt_bias, a, d, q_start, q_len, ctx_len, state_slot, groups, num_seqs):
    H, V, N = state.shape[1:]
    taps, C = conv_w.shape
    R, inner = ring.shape[1], H * V
    for s in range(num_seqs):
        n, q0, slot = int(q_len[s]), int(q_start[s]), int(state_slot[s])
        if n <= 0:
            continue
        p0 = int(ctx_len[s]) - n
        rows = proj[q0:q0 + n]
        xin = rows[:, inner:inner + C].float()
        before = [ring[slot, p % R].float() if p >= 0 else torch.zeros(C) for p in range(p0 - taps + 1, p0)]
        full = torch.cat([torch.stack(before), xin]) if before else xin
        u = conv_b + sum(full[k:k + n] * conv_w[k] for k in range(taps))
        u = (u * torch.sigmoid(u)).to(proj.dtype).float()
        for p in range(max(p0, p0 + n - taps + 1), p0 + n):
            ring[slot, p % R] = rows[p - p0, inner:inner + C]
        x, B, Cm = u[:, :inner].view(n, H, V), u[:, inner:inner + groups * N], u[:, inner + groups * N:]
        B = B.view(n, groups, N).repeat_interleave(H // groups, 1)
        Cm = Cm.view(n, groups, N).repeat_interleave(H // groups, 1)
        dt = rows[:, inner + C:inner + C + H].float() + dt_bias
        dt = dt.clamp(min=0) + torch.log1p(torch.exp(-dt.abs()))
        S = state[slot].clone() if p0 > 0 else torch.zeros(H, V, N)
        for t in range(n):
            S = S * torch.exp(-a * dt[t])[:, None, None] + (dt[t][:, None] * x[t])[:, :, None] * B[t][:, None, :]
            o = (S * Cm[t][:, None, :]).sum(-1) + d[:, None] * x[t]
            y[q0 + t, :inner] = o.reshape(-1).to(y.dtype)
        state[slot] = S


def matrix_memory(x, y, div, state, top, i_bias, f_bias, q_start, q_len, ctx_len, state_slot, cols, vdim, cap, q_scale,
                  num_seqs):
    H, V, N = state.shape[1:]
    cq, ck, cv, ci, vin = cols
    for s in range(num_seqs):
        n, q0, slot = int(q_len[s]), int(q_start[s]), int(state_slot[s])
        if n <= 0:
            continue
        r = x[q0:q0 + n].float()
        q, k = r[:, cq:cq + H * N].view(n, H, N) * q_scale, r[:, ck:ck + H * N].view(n, H, N)
        v = torch.zeros(n, H, V)
        v[:, :, :vdim] = r[:, cv:cv + H * vin].view(n, H, vin)[:, :, :vdim]
        v[:, :, vdim] = 1.0  # (the row that sums the keys)
        i = cap * torch.tanh((r[:, ci:ci + H] + i_bias) / cap)
        f = torch.nn.functional.logsigmoid(cap * torch.tanh((r[:, ci + H:ci + 2 * H] + f_bias) / cap))
        fresh = int(ctx_len[s]) == n
        S, m = (torch.zeros(H, V, N), torch.zeros(H)) if fresh else (state[slot].clone(), top[slot, :, 0].clone())
        for t in range(n):
            mn = torch.maximum(f[t] + m, i[t])
            S = S * torch.exp(f[t] + m - mn)[:, None, None] + \
                (torch.exp(i[t] - mn)[:, None] * v[t])[:, :, None] * k[t][:, None, :]
            m = mn
            o = (S * q[t][:, None, :]).sum(-1)
            y[q0 + t, :H * vin].view(H, vin)[:, :vdim] = o[:, :vdim].to(y.dtype)
            div[q0 + t] = torch.maximum(o[:, vdim].abs(), torch.exp(-m)) + 1e-6
        state[slot], top[slot] = S, m[:, None]


def linear_attention(x, y, state, a2, bias, q_start, q_len, ctx_len, state_slot, cols, q_scale, inv_tau, num_seqs):
    H, V, N = state.shape[1:]
    cq, ck, cv, ca = cols
    for s in range(num_seqs):
        n, q0, slot = int(q_len[s]), int(q_start[s]), int(state_slot[s])
        if n <= 0:
            continue
        r = x[q0:q0 + n].float()
        q, k = r[:, cq:cq + H * N].view(n, H, N) * q_scale, r[:, ck:ck + H * N].view(n, H, N)
        v = r[:, cv:cv + H * V].view(n, H, V)
        z = r[:, ca:ca + a2.shape[1]] @ a2.float().T + bias
        d = torch.exp(torch.nn.functional.logsigmoid(z) * inv_tau).view(n, H, 1, N)
        S = torch.zeros(H, V, N) if int(ctx_len[s]) == n else state[slot].clone()
        for t in range(n):
            S = S * d[t] + v[t][:, :, None] * k[t][:, None, :]
            y[q0 + t, :H * V] = (S * q[t][:, None, :]).sum(-1).reshape(-1).to(y.dtype)
        state[slot] = S


def poly_norm(z, n, act, eps):
    f = z[:, :n].float()
    z[:, :n] = (sum(act[i] * _norm32(f ** (i + 1), eps) for i in range(3)) + act[3]).to(z.dtype)
    z[:, n:] = 0


def gated_norm(y, z, w, heads, vdim, vpad, parts, eps, div, after):
    T = y.shape[0]
    g, zf = (t[:, :heads * vpad].float().reshape(T, heads, vpad)[:, :, :vdim] for t in (y, z))
    if div is not None:
        g = g / div[:, :, None]
    g, zf = g.reshape(T, -1), zf.reshape(T, -1)
    if after is None:
        g = g * (zf * torch.sigmoid(zf))
    g = _norm32(g.view(T, parts, -1), eps).view(T, -1) * w
    if after is not None:
        g = g * torch.sigmoid(zf) * (zf if after == "silu" else 1.0)
    y.zero_()
    y[:, :heads * vpad].view(T, heads, vpad)[:, :, :vdim] = g.view(T, heads, vdim).to(y.dtype)


def score_route(h, w, slots, weights, choice, order, tiles, n_tiles, E, top, groups, keep, always, tm, softmax, correction,
                share, scale):
    T = h.shape[0]
    z = h[:, :w.shape[1]].float() @ w[:E].float().T
    s = torch.softmax(z, -1) if softmax else torch.sigmoid(z)
    pick = s + correction if correction is not None else s
    per = pick.view(T, groups, E // groups)
    best = per.topk(min(2, E // groups), -1).values.sum(-1).topk(keep, -1).indices
    ok = torch.zeros(T, groups, dtype=torch.bool).scatter_(1, best, True).repeat_interleave(E // groups, 1)
    idx = pick.masked_fill(~ok, float("-inf")).topk(top, -1).indices
    val = s.gather(1, idx)
    if share:
        val = val / (val.sum(1, keepdim=True) + 1e-20)
    live = slots[:T] >= 0
    weights[:, :top], weights[:, top:] = val * scale, 1.0
    weights[~live] = 0
    e = torch.cat([idx, torch.arange(E, E + always).expand(T, -1)], 1)
    choice.view(T, top + always).copy_(torch.where(live[:, None], e, -1))
    p = torch.arange(T * (top + always))[live.repeat_interleave(top + always)]
    ep = e.reshape(-1)[p]
    p = p[torch.argsort(ep, stable=True)]
    order[:len(p)] = p.to(torch.int32)
    k, start = 0, 0
    for x, c in enumerate(torch.bincount(ep, minlength=E + always).tolist()):
        for i in range(0, c, tm):
            tiles[k] = torch.tensor([x, start + i, min(tm, c - i), 0], dtype=torch.int32)
            k += 1
        start += c
    n_tiles[0] = k
