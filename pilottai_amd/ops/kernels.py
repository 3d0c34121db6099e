"""Dispatch layer for the CDNA4 HIP kernels (pilottai_amd/_C.so).

Device tensors ALWAYS go to the native kernels: if the extension failed to load
on a machine with a GPU, every call raises (no silent PyTorch fallback — the
round-end driver checks which .so files the GPU tests actually loaded). CPU
tensors run the fp32 reference implementations in ops/reference.py, which is
how the control-plane tests execute the whole engine without a GPU.
"""
from __future__ import annotations

import importlib
import os
from typing import Optional

import torch

from . import reference as ref

_C = None
_LOAD_ERROR: Optional[BaseException] = None


def _load():
    global _C, _LOAD_ERROR
    if _C is not None or _LOAD_ERROR is not None:
        return _C
    try:
        _C = importlib.import_module("pilottai_amd._C")
        if os.environ.get("PILOTTAI_DECODE_VARIANT"):  # A/B switch of the packed decode GEMM
            _C.decode_set_variant(int(os.environ["PILOTTAI_DECODE_VARIANT"]))
    except BaseException as e:  # noqa: BLE001 — surfaced by require_native()
        _LOAD_ERROR = e
    return _C


def native_available() -> bool:
    return _load() is not None


def require_native():
    mod = _load()
    if mod is None:
        raise RuntimeError(
            "pilottai_amd native kernels (_C.so) are not available: "
            f"{_LOAD_ERROR!r}. Build them with `python -m pilottai_amd._build` "
            "(hipcc --offload-arch=gfx950).")
    return mod


_FAMILY = {}


def _require_family(name: str):
    if name not in _FAMILY:
        try:
            _FAMILY[name] = importlib.import_module("pilottai_amd._" + name)
        except ImportError as e:
            raise RuntimeError(f"pilottai_amd {name} kernels (_{name}.so) are not available: {e!r}. Build them with "
                               "`python -m pilottai_amd._build` (hipcc --offload-arch=gfx950).") from e
    return _FAMILY[name]


# the modules that hold an operation, by what they are built for (_build.py MODULES)
LATENT = ("latent", "latent_linear")
MIXED = ("hybrid", "latent_linear")
GROUPED = ("latent", "hybrid", "latent_linear")


def require_family(*names: str):
    """Of these modules the one that a model has loaded, else the first that is built."""
    for name in _FAMILY:
        if name in names:
            return _FAMILY[name]
    for name in names[:-1]:
        try:
            return _require_family(name)
        except RuntimeError:
            pass
    return _require_family(names[-1])


def require_latent():
    """A module with latent attention and its residual (csrc/ops/bind_latent.h)."""
    return require_family(*LATENT)


def require_hybrid():
    """The _hybrid module (paged attention, recurrent layers, score-routed experts, fp32 residuals;
    csrc/ops/bindings_hybrid.cpp)."""
    return require_family("hybrid")


def require_grouped():
    """A module with the grouped projections."""
    return require_family(*GROUPED)


def _packed_module():
    """The module with the packed-weight projections: _C, or a family's where only that one is built."""
    return _load() or require_grouped()


def native_module_path() -> Optional[str]:
    mod = _load()
    return getattr(mod, "__file__", None) if mod is not None else None


def _on_gpu(t: torch.Tensor) -> bool:
    return t.device.type == "cuda"


# ---------------------------------------------------------------------------


def empty_handoff(numel: int, dtype=torch.float32, device=None) -> torch.Tensor:
    """A buffer that one workgroup writes and another reads INSIDE one launch (split-K slabs,
    attention partition partials). On the GPU it lives in uncached device memory
    (hipDeviceMallocUncached): no CU or XCD can hold a stale copy of its lines, so the
    in-launch hand-off is correct for any workgroup placement with a relaxed ticket and the
    last arriver's acquire, and needs no producer-side L2 write-back (
    profiles/r4_handoff_uncached.md). Zero-filled. Allocate outside graph capture."""
    device = torch.device(device) if device is not None else torch.device("cpu")
    if device.type == "cuda":
        idx = device.index if device.index is not None else torch.cuda.current_device()
        return _packed_module().empty_uncached(int(numel), dtype, int(idx))
    return torch.zeros(int(numel), dtype=dtype, device=device)


def rmsnorm(x: torch.Tensor, w: torch.Tensor, eps: float, out: Optional[torch.Tensor] = None):
    if _on_gpu(x):
        out = torch.empty_like(x) if out is None else out
        require_native().rmsnorm(out, x, w, float(eps))
        return out
    r = ref.rmsnorm(x, w, eps)
    if out is not None:
        out.copy_(r)
        return out
    return r


def fused_add_rmsnorm(resid: torch.Tensor, x: torch.Tensor, w: torch.Tensor, eps: float,
                      out: Optional[torch.Tensor] = None):
    """resid <- resid + x (in place); returns rmsnorm(resid) * w."""
    if _on_gpu(x):
        out = torch.empty_like(x) if out is None else out
        require_native().fused_add_rmsnorm(out, resid, x, w, float(eps))
        return out
    y, nr = ref.fused_add_rmsnorm(resid, x, w, eps)
    resid.copy_(nr)
    if out is not None:
        out.copy_(y)
        return out
    return y


def silu_mul(x: torch.Tensor, out: Optional[torch.Tensor] = None):
    if _on_gpu(x):
        F = x.shape[-1] // 2
        out = torch.empty(*x.shape[:-1], F, dtype=x.dtype, device=x.device) if out is None else out
        require_native().silu_mul(out, x)
        return out
    r = ref.silu_mul(x)
    if out is not None:
        out.copy_(r)
        return out
    return r


def rope_cache(q_out, k_cache, v_cache, qkv, positions, slot_mapping, cos_sin, H: int, KV: int,
               apply_rope: bool = True):
    if _on_gpu(qkv):
        require_native().rope_cache(q_out, k_cache, v_cache, qkv, positions, slot_mapping, cos_sin,
                                    int(H), int(KV), bool(apply_rope))
        return q_out
    ref.rope_cache(q_out, k_cache, v_cache, qkv, positions, slot_mapping, cos_sin, H, KV,
                   apply_rope)
    return q_out


def paged_attention(out, part_o, part_ml, q, k_cache, v_cache, items, n_items, counters,
                    q_start, q_len, ctx_len, block_table, scale: float, num_seqs: Optional[int] = None,
                    part_size: Optional[torch.Tensor] = None, waves: int = 4):
    """Attention over the paged cache. On GPU `items` must be a device int32
    [max, 4] tensor with a device count (graph-capturable) and `counters` a
    zero-initialised int32 tensor of >= seqs * KV entries (partition tickets; the
    kernel leaves it zeroed); on CPU the reference path ignores both. `waves` 8: 512-thread workgroups for the decode and 32-column prefill items (small decode
    batches; wide items run as their 32-column sub-items)."""
    if _on_gpu(q):
        require_native().paged_attention(out, part_o, part_ml, q, k_cache, v_cache, items, n_items,
                                         counters, q_start, q_len, ctx_len, block_table,
                                         float(scale), part_size, int(waves))
        return out
    ns = len(q_len) if num_seqs is None else num_seqs
    r = ref.paged_attention(q, k_cache, v_cache, q_start[:ns], q_len[:ns], ctx_len[:ns],
                            block_table, scale)
    n_tok = int(q_start[ns - 1] + q_len[ns - 1]) if ns > 0 else 0
    out[:n_tok].copy_(r[:n_tok])
    return out


def sample_workspace(rows: int, V: int, device) -> torch.Tensor:
    n = require_native().sample_workspace_floats(rows, V)
    return torch.empty(n, dtype=torch.float32, device=device)


def topkp_threshold(logits, V: int, temperature, top_k, top_p, mask_class, class_masks,
                    out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Per-row logit threshold tau for top-k / top-p (csrc/ops/sampling.hip).

    `logits` is [rows, V] or a TP all-gather [shards, rows, V/shards]."""
    rows = logits.shape[-2]
    tau = out if out is not None else torch.empty(rows, dtype=torch.float32, device=logits.device)
    if _on_gpu(logits):
        require_native().topkp_threshold(tau, logits, int(V), temperature, top_k, top_p, mask_class,
                                         class_masks)
        return tau
    full = logits if logits.dim() == 2 else logits.permute(1, 0, 2).reshape(rows, V)
    tau[:rows].copy_(ref.topkp_threshold(full, temperature, top_k, top_p, mask_class, class_masks))
    return tau


def patch_pending_ids(ids: torch.Tensor, sampled: torch.Tensor) -> None:
    """In place: ids[t] = sampled[-ids[t] - 1] where ids[t] < 0 (pipelined engine steps:
    a row's pending token comes from the previous step's sampler, csrc/ops/sampling.hip)."""
    if _on_gpu(ids):
        require_native().patch_pending_ids(ids, sampled)
        return
    neg = ids < 0
    if bool(neg.any()):
        r = (-ids[neg] - 1).long()
        ids[neg] = torch.where(r < sampled.numel(), sampled[r.clamp(max=sampled.numel() - 1)],
                               torch.zeros_like(r, dtype=ids.dtype))


def sample(logits, temperature, mask_class, class_masks, seeds, offsets, forced=None,
           out: Optional[torch.Tensor] = None, workspace: Optional[torch.Tensor] = None,
           vocab_offset: int = 0, out_keys: Optional[torch.Tensor] = None,
           tau: Optional[torch.Tensor] = None):
    rows = logits.shape[0]
    if _on_gpu(logits):
        C = require_native()
        out = torch.empty(rows, dtype=torch.int32, device=logits.device) if out is None else out
        if workspace is None:
            workspace = sample_workspace(rows, logits.shape[1], logits.device)
        C.sample(out, out_keys, workspace, logits, int(vocab_offset), temperature, mask_class,
                 class_masks, seeds, offsets, forced, tau)
        return out
    toks, keys = ref.sample(logits, temperature, mask_class, class_masks, seeds, offsets, forced,
                            vocab_offset, return_keys=True, tau=tau)
    if out_keys is not None:
        out_keys[:rows].copy_(keys)
    if out is not None:
        out[:rows].copy_(toks)
        return out
    return toks


COSINE_MAX_Q = 64  # queries per index pass (LDS-resident query tiles)


def cosine_topk(queries, index, n_valid: int, K: int, row_priority, row_tags, row_expiry,
                q_min_priority, q_tags, now: float, workspace: Optional[torch.Tensor] = None):
    if _on_gpu(index):
        C = require_native()
        Q = queries.shape[0]
        out_s = torch.empty(Q, K, dtype=torch.float32, device=index.device)
        out_r = torch.empty(Q, K, dtype=torch.int32, device=index.device)
        qc = min(Q, COSINE_MAX_Q)
        need = C.cosine_topk_workspace_bytes(qc, max(1, int(n_valid)), K)
        if workspace is None or workspace.numel() * workspace.element_size() < need:
            workspace = torch.empty(max(need, 16), dtype=torch.uint8, device=index.device)
        # one pass over the index per <= 64 queries (csrc/ops/similarity.hip)
        for q0 in range(0, Q, COSINE_MAX_Q):
            q1 = min(Q, q0 + COSINE_MAX_Q)
            C.cosine_topk(out_s[q0:q1], out_r[q0:q1], workspace, queries[q0:q1].contiguous(), index,
                          int(n_valid), int(K), row_priority, row_tags, row_expiry,
                          q_min_priority[q0:q1].contiguous(), q_tags[q0:q1].contiguous(), float(now))
        return out_s, out_r
    if index.dim() == 4:  # packed tiles (memory/semantic_index.py) -> row-major for the reference
        index = unpack_decode_weight(index)
    return ref.cosine_topk(queries, index, n_valid, K, row_priority, row_tags, row_expiry,
                           q_min_priority, q_tags, now)


# ---- 16-bit fixed-point index (csrc/ops/similarity_q16.hip; memory/semantic_index.py storage="q16")
Q16_MAX = 32512  # |v| <= 127 * 256: hi = floor((v + 128) / 256) stays in [-127, 127]


def q16_quantize(x: torch.Tensor):
    """Rows of x (any float) -> (hi int8 [n, D], lo int8 [n, D], scale fp32 [n], bound fp32 [n]):
    v = round(x / scale) = 256 hi + lo exactly (|v| <= Q16_MAX, scale = max|x| / Q16_MAX), and
    bound = scale * ||lo||_2 (a hair above: the stage-1 error bound's row factor)."""
    x = x.float()
    m = x.abs().amax(1)
    sc = torch.where(m > 0, m / Q16_MAX, torch.ones_like(m))
    v = torch.round(x / sc[:, None]).clamp_(-Q16_MAX, Q16_MAX)
    hi = torch.floor((v + 128) / 256)
    lo = v - 256 * hi
    bound = (sc.double() * lo.double().norm(dim=1)).float() * (1 + 1e-6)
    return hi.to(torch.int8), lo.to(torch.int8), sc, bound


def q16_pack(plane: torch.Tensor) -> torch.Tensor:
    """int8 [n = 16 T, D] -> fragment-major tiles [T, D/64, 64, 16]: lane 16 g + c of (t, s) holds
    row 16 t + c, dims 64 s + 16 g .. + 16 (the v_mfma_i32_16x16x64_i8 operand)."""
    n, D = plane.shape
    return plane.reshape(n // 16, 16, D // 64, 4, 16).permute(0, 2, 3, 1, 4).reshape(n // 16, D // 64, 64, 16)


def q16_unpack(tiles: torch.Tensor) -> torch.Tensor:
    T, DS = tiles.shape[0], tiles.shape[1]
    return tiles.view(T, DS, 4, 16, 16).permute(0, 3, 1, 2, 4).reshape(T * 16, DS * 64)


def q16_queries(q: torch.Tensor):
    """Queries -> (qv int8 [Q, 2, D] = (qh, ql), qmeta fp32 [Q, 2] = (scale, scale * ||v||_2))."""
    hi, lo, sc, _ = q16_quantize(q)
    v = 256 * hi.double() + lo.double()
    cq = (sc.double() * v.norm(dim=1)).float() * (1 + 1e-6)
    return torch.stack([hi, lo], 1).contiguous(), torch.stack([sc, cq], 1).contiguous()


def q16_topk(queries, hi, lo, rmeta, n_valid: int, K: int, row_priority, row_tags, row_expiry,
             q_min_priority, q_tags, now: float, workspace: Optional[torch.Tensor] = None, exact: bool = False,
             stats: Optional[dict] = None):
    """Exact filtered top-k over a q16 index (scores of the 16-bit fixed-point vectors, the
    same on the GPU and in ops.reference.q16_topk). GPU: the two-stage kernel, hi plane only in
    the streaming pass; a batch whose drop check fails is re-run with the exact scan (counted
    in stats["q16_fallbacks"]). queries: fp32 / bf16 [Q, D] (quantised here)."""
    qv, qm = q16_queries(queries)
    if _on_gpu(hi):
        C = require_native()
        Q = qv.shape[0]
        out_s = torch.empty(Q, K, dtype=torch.float32, device=hi.device)
        out_r = torch.empty(Q, K, dtype=torch.int32, device=hi.device)
        unsafe = torch.zeros(Q, dtype=torch.int32, device=hi.device)
        qc = min(Q, COSINE_MAX_Q)
        need = C.q16_topk_workspace_bytes(qc, max(1, int(n_valid)))
        if workspace is None or workspace.numel() * workspace.element_size() < need:
            workspace = torch.empty(max(need, 16), dtype=torch.uint8, device=hi.device)
        for q0 in range(0, Q, COSINE_MAX_Q):
            q1 = min(Q, q0 + COSINE_MAX_Q)
            C.q16_topk(out_s[q0:q1], out_r[q0:q1], unsafe[q0:q1], workspace, qv[q0:q1], qm[q0:q1], hi, lo, rmeta,
                       int(n_valid), int(K), row_priority, row_tags, row_expiry,
                       q_min_priority[q0:q1].contiguous(), q_tags[q0:q1].contiguous(), float(now), int(exact))
        if not exact and bool(unsafe.any()):  # a slice refused a row that might be in the top-k
            if stats is not None:
                stats["q16_fallbacks"] = stats.get("q16_fallbacks", 0) + 1
            for q0 in range(0, Q, COSINE_MAX_Q):
                q1 = min(Q, q0 + COSINE_MAX_Q)
                C.q16_topk(out_s[q0:q1], out_r[q0:q1], unsafe[q0:q1], workspace, qv[q0:q1], qm[q0:q1], hi, lo,
                           rmeta, int(n_valid), int(K), row_priority, row_tags, row_expiry,
                           q_min_priority[q0:q1].contiguous(), q_tags[q0:q1].contiguous(), float(now), 1)
        return out_s, out_r
    return ref.q16_topk(qv, qm, hi, lo, rmeta, n_valid, K, row_priority, row_tags, row_expiry,
                        q_min_priority, q_tags, now)


def skinny_gemm(x: torch.Tensor, w: torch.Tensor, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """y = x @ w.T via the weight-streaming MFMA kernel (csrc/ops/gemm_skinny.hip)."""
    y = out if out is not None else torch.empty(x.shape[0], w.shape[0], dtype=x.dtype, device=x.device)
    if not _on_gpu(x):
        y.copy_(torch.nn.functional.linear(x.float(), w.float()).to(y.dtype))
        return y
    if not require_native().skinny_gemm(y, x, w):
        raise ValueError(f"skinny_gemm does not handle M={x.shape[0]} N={w.shape[0]} K={x.shape[1]}")
    return y


# Largest token count at which the skinny kernel beats hipBLASLt, per projection
# kind, measured cache-cold on MI355X with Llama-3-8B shapes
# (tools/gemm_bench.py, profiles/r1_skinny_gemm_cold.md). 0 = never.
SKINNY_MAX_M = {"qkv": 8, "o": 32, "gate_up": 16, "down": 0, "lm_head": 0}


def linear(x: torch.Tensor, w: torch.Tensor, kind: str) -> torch.Tensor:
    """Projection dispatcher: skinny MFMA kernel at decode sizes, hipBLASLt otherwise.

    The choice depends only on the (static) token count, so it is fixed per
    captured hipGraph bucket."""
    M, K = x.shape
    if (_on_gpu(x) and M <= SKINNY_MAX_M.get(kind, 0) and K % 256 == 0 and w.shape[0] % 16 == 0
            and x.is_contiguous()):
        return skinny_gemm(x, w)
    return torch.nn.functional.linear(x, w)


# ---------------------------------------------------------------------------
# Decode-step projections on fragment-major packed weights (csrc/ops/gemm_decode.hip)

DECODE_EPI = {"plain": 0, "silu": 1, "resid": 2}


def pack_decode_weight(w: torch.Tensor) -> torch.Tensor:
    """[N, K] row-major -> [N/16, K/32, 64, 8]: lane l = 16*g + c of tile (t, s)
    holds w[16t + c, 32s + 8g : 32s + 8g + 8] (the MFMA 16x16x32 B fragment)."""
    N, K = w.shape
    if N % 16 or K % 32:
        raise ValueError(f"cannot pack a [{N}, {K}] weight (needs N % 16 == 0, K % 32 == 0)")
    return w.reshape(N // 16, 16, K // 32, 4, 8).permute(0, 2, 3, 1, 4).contiguous().view(N // 16, K // 32, 64, 8)


def pack_decode_gate_up(w13: torch.Tensor) -> torch.Tensor:
    """[2F, K] = [gate; up] -> packed tiles interleaved (gate t, up t, gate t+1, ...),
    so one workgroup holds both halves of the same 16 outputs (EPI silu)."""
    F2, K = w13.shape
    F = F2 // 2
    g = pack_decode_weight(w13[:F])
    u = pack_decode_weight(w13[F:])
    return torch.stack([g, u], 1).reshape(F2 // 16, K // 32, 64, 8)


def unpack_decode_weight(wp: torch.Tensor) -> torch.Tensor:
    T, S = wp.shape[0], wp.shape[1]
    return wp.view(T, S, 4, 16, 8).permute(0, 3, 1, 2, 4).reshape(T * 16, S * 32)


def unpack_decode_gate_up(wp: torch.Tensor) -> torch.Tensor:
    T, S = wp.shape[0], wp.shape[1]
    pairs = wp.view(T // 2, 2, S, 64, 8)
    return torch.cat([unpack_decode_weight(pairs[:, 0]), unpack_decode_weight(pairs[:, 1])], 0)


def decode_gemm(x: torch.Tensor, wp: torch.Tensor, epi: str = "plain", norm: bool = False,
                eps: float = 1e-5, resid: Optional[torch.Tensor] = None,
                out: Optional[torch.Tensor] = None, nt: int = 0, waves: int = 0, splits: int = 0) -> torch.Tensor:
    """y = epi(rownorm(x) @ W.T) for M <= 64 rows with W packed by pack_decode_weight
    (gate_up: pack_decode_gate_up). `norm` scales each row by rsqrt(mean(x^2)+eps)
    (the RMSNorm weight must already be folded into W); epi "silu" returns
    silu(gate)*up [M, F]; epi "resid" returns resid + acc (out may alias resid)."""
    M, K = x.shape
    N = wp.shape[0] * 16
    code = DECODE_EPI[epi]
    NO = N // 2 if code == 1 else N
    if out is None:
        out = torch.empty(M, NO, dtype=x.dtype, device=x.device)
    if _on_gpu(x):
        ws, cnt = decode_workspace(x.device)
        if not _packed_module().decode_gemm(out, x, wp, resid, code, bool(norm), float(eps), int(nt), int(waves),
                                            int(splits), ws, cnt):
            raise ValueError(f"decode_gemm does not handle M={M} N={N} K={K} epi={epi} nt={nt} waves={waves}")
        return out
    xf = x.float()
    W = unpack_decode_gate_up(wp) if code == 1 else unpack_decode_weight(wp)
    acc = xf @ W.float().T
    if norm:
        acc = acc * torch.rsqrt(xf.pow(2).mean(-1, keepdim=True) + eps)
    if code == 1:
        g, u = acc[:, :NO], acc[:, NO:]
        acc = g * torch.sigmoid(g) * u
    elif code == 2:
        acc = acc + resid.float()
    out.copy_(acc.to(out.dtype))
    return out


# per-head tile order of the rope-fused QKV weights: tiles (i, i + 4) adjacent
_ROPE_TILE_ORDER = (0, 4, 1, 5, 2, 6, 3, 7)


def pack_decode_qkv_rope(wqkv: torch.Tensor) -> torch.Tensor:
    """Packed QKV weights for decode_qkv_rope: within every 128-row head the
    16-row tiles are reordered to (0, 4, 1, 5, 2, 6, 3, 7), so one workgroup of
    two tiles holds rotary dims i and i + 64 (csrc/ops/gemm_decode.hip EPI_ROPE)."""
    N, K = wqkv.shape
    if N % 128:
        raise ValueError("QKV rows must be a multiple of the 128-wide head")
    idx = torch.tensor(_ROPE_TILE_ORDER, device=wqkv.device)
    w = wqkv.reshape(N // 128, 8, 16, K).index_select(1, idx).reshape(N, K)
    return pack_decode_weight(w)


def unpack_decode_qkv_rope(wp: torch.Tensor) -> torch.Tensor:
    w = unpack_decode_weight(wp)
    N, K = w.shape
    inv = torch.argsort(torch.tensor(_ROPE_TILE_ORDER)).to(w.device)
    return w.reshape(N // 128, 8, 16, K).index_select(1, inv).reshape(N, K)


def decode_qkv_rope(x: torch.Tensor, wp: torch.Tensor, eps: float, q_out: torch.Tensor, k_cache, v_cache,
                    positions, slots, cos_sin, H: int, KV: int, splits: int = 0) -> torch.Tensor:
    """Decode QKV projection with the RMSNorm folded in (norm weight pre-multiplied
    into the packed weights), RoPE and the paged KV write fused in the epilogue:
    replaces rmsnorm + QKV GEMM + rope_cache on decode-sized steps."""
    if _on_gpu(x):
        ws, cnt = decode_workspace(x.device)
        require_native().decode_qkv_rope(x, wp, float(eps), q_out, k_cache, v_cache, positions, slots,
                                         cos_sin, int(H), int(KV), int(splits), ws, cnt)
        return q_out
    xf = x.float()
    w = unpack_decode_qkv_rope(wp).float()
    qkv = (xf @ w.T) * torch.rsqrt(xf.pow(2).mean(-1, keepdim=True) + eps)
    ref.rope_cache(q_out, k_cache, v_cache, qkv.to(x.dtype), positions, slots, cos_sin, H, KV)
    return q_out


# split-K slabs + tickets of the packed decode kernels (decode_gemm / decode_qkv_rope)
DECODE_WS_FLOATS = 8 << 20  # 32 MB of split-K slabs per device
_decode_ws = {}


def decode_workspace(device):
    """(slabs, tickets) for decode_gemm / decode_qkv_rope on `device`; allocate before
    hipGraph capture (the tickets must start zeroed; every launch leaves them zeroed)."""
    key = str(device)
    if key not in _decode_ws:
        _decode_ws[key] = (empty_handoff(DECODE_WS_FLOATS, torch.float32, device),
                           torch.zeros(16384, dtype=torch.int32, device=device))
    return _decode_ws[key]


# ---------------------------------------------------------------------------
# Mid-size projections (48 < M <= 512) on the packed weights (csrc/ops/gemm_mid.hip)

MID_EPI = {"plain": 0, "silu": 1, "resid": 2, "rope_perm": 3}
MID_WS_FLOATS = 16 << 20  # 64 MB of split-K slabs per device
_mid_ws = {}


def mid_workspace(device):
    """(slabs, tickets) for mid_gemm / mid_qkv_rope on `device`; allocate before hipGraph
    capture (the tickets start zeroed and every launch leaves them zeroed)."""
    key = str(device)
    if key not in _mid_ws:
        _mid_ws[key] = (empty_handoff(MID_WS_FLOATS, torch.float32, device),
                        torch.zeros(16384, dtype=torch.int32, device=device))
    return _mid_ws[key]


def _unpack_for(code: int, wp: torch.Tensor) -> torch.Tensor:
    if code == 3:
        return unpack_decode_qkv_rope(wp)
    if code == 1:
        return unpack_decode_gate_up(wp)
    return unpack_decode_weight(wp)


def row_sumsq(x: torch.Tensor, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """out[m] = sum_k x[m, k]^2 in fp32 (RMSNorm row statistics)."""
    out = torch.empty(x.shape[0], dtype=torch.float32, device=x.device) if out is None else out
    if _on_gpu(x):
        require_native().row_sumsq(out, x)
        return out
    out[:x.shape[0]].copy_(x.float().pow(2).sum(-1))
    return out


def mid_gemm(x: torch.Tensor, wp: torch.Tensor, epi: str = "plain", resid: Optional[torch.Tensor] = None,
             out: Optional[torch.Tensor] = None, norm: bool = False, eps: float = 1e-5, fm: int = 0, fn: int = 0,
             splits: int = 0, ss_in: Optional[torch.Tensor] = None, ss_out: Optional[torch.Tensor] = None,
             ss_zero: Optional[torch.Tensor] = None) -> torch.Tensor:
    """y = epi(rownorm(x) @ W.T) for mid-size M with W packed by pack_decode_weight (gate_up:
    pack_decode_gate_up + epi "silu"; QKV: pack_decode_qkv_rope + epi "rope_perm", which
    returns the natural column order); "resid": resid + acc (out may alias resid).

    `norm` scales rows by rsqrt(mean(x^2) + eps) (RMSNorm weight folded into W); the row
    statistics are `ss_in` ([M] fp32 sum of x^2, e.g. the `ss_out` of the residual epilogue
    that produced x) or computed here by row_sumsq. `ss_out` (resid only): [M] += row sums
    of the written output squared. `ss_zero`: an [M] buffer zeroed by the launch."""
    M, K = x.shape
    N = wp.shape[0] * 16
    code = MID_EPI[epi]
    NO = N // 2 if code == 1 else N
    if out is None:
        out = torch.empty(M, NO, dtype=x.dtype, device=x.device)
    if norm and ss_in is None:
        ss_in = row_sumsq(x)
    if _on_gpu(x):
        ws, cnt = mid_workspace(x.device)
        if not require_native().mid_gemm(out, x, wp, resid, ws, cnt, code, ss_in if norm else None, ss_out, ss_zero,
                                          float(eps), int(fm), int(fn), int(splits)):
            raise ValueError(f"mid_gemm does not handle M={M} N={N} K={K} epi={epi} fm={fm} fn={fn} S={splits}")
        return out
    W = _unpack_for(code, wp)
    acc = x.float() @ W.float().T
    if norm:
        acc = acc * torch.rsqrt(ss_in[:M].float().unsqueeze(-1) / K + eps)
    if code == 1:
        acc = torch.nn.functional.silu(acc[:, :NO]) * acc[:, NO:]
    elif code == 2:
        acc = acc + resid.float()
    y = acc.to(out.dtype)
    if ss_zero is not None:
        ss_zero[:M].zero_()
    if ss_out is not None:
        ss_out[:M] += y.float().pow(2).sum(-1)
    out.copy_(y)
    return out


# ---------------------------------------------------------------------------
# Weight-streaming projections (16 < M <= 256) on the packed weights (csrc/ops/gemm_stream.hip)

STREAM_EPI = {"plain": 0, "silu": 1, "resid": 2, "rope_perm": 3}
STREAM_WS_FLOATS = 24 << 20  # 96 MB of split-K partial fragments per device (uncached)
_stream_ws = {}
# Split-K group hand-off of gemm_stream.hip (rel bit 0 = the producer's agent-scope release,
# buffer_wbl2 sc1 + drain, before it arrives). Shipped: 0, the form of MI355X_MICROARCH.md's
# measured-valid hand-off table, row 1 (16-B sc1 slab stores drained by every wave, workgroup
# barrier, one lane's agent-scope add; sc1 poll; sc1 slab loads behind a barrier), plus the
# consumer's agent-scope acquire. Round 5 ran 100,000 NaN-poisoned, varied-input repetitions of
# every production plan (the RoPE + paged-KV epilogue included) in both forms: 0 bad runs
# (profiles/r5_handoff_stream.md); the release costs 2.5-5 us per launch (+10-18 %, about +5 %
# on a 64-row step), so it stays an option (PILOTTAI_STREAM_REL=1). The decode / mid / prefill
# last-arriver hand-offs keep their release (they failed without it, profiles/r4_handoff_uncached.md).
STREAM_REL = int(os.environ.get("PILOTTAI_STREAM_REL", "0"))


def stream_workspace(device):
    """(slabs, counters, err) for stream_gemm / stream_qkv_rope on `device`; allocate before
    hipGraph capture. Slabs live in uncached memory (empty_handoff); the group counters start
    zeroed and every launch leaves them zeroed; err[0] != 0 means a group barrier timed out."""
    key = str(device)
    if key not in _stream_ws:
        _stream_ws[key] = (empty_handoff(STREAM_WS_FLOATS, torch.float32, device),
                           torch.zeros(16384, dtype=torch.int32, device=device),
                           torch.zeros(16, dtype=torch.int32, device=device))
    return _stream_ws[key]


def stream_gemm_plan(M: int, N: int, K: int, epi: str = "plain"):
    """Default decomposition (mg, rg, tpw, wt, wk, S, D) of stream_gemm for this shape."""
    code = 4 if epi == "rope_kv" else STREAM_EPI[epi]
    return tuple(require_native().stream_gemm_plan(int(M), int(N), int(K), code)[:7])


def stream_gemm(x: torch.Tensor, wp: torch.Tensor, epi: str = "plain", resid: Optional[torch.Tensor] = None,
                out: Optional[torch.Tensor] = None, norm: bool = False, eps: float = 1e-5,
                ss_in: Optional[torch.Tensor] = None, ss_out: Optional[torch.Tensor] = None,
                ss_zero: Optional[torch.Tensor] = None, plan=None, rel: Optional[int] = None,
                stamps: Optional[torch.Tensor] = None) -> torch.Tensor:
    """y = epi(rownorm(x) @ W.T) for 16 < M <= 256 with W packed by pack_decode_weight (gate_up:
    pack_decode_gate_up + "silu"; QKV: pack_decode_qkv_rope + "rope_perm"); same epilogue and
    row-statistics conventions as mid_gemm. `plan`: (mg, rg, tpw, wt, wk, S, D) or None for
    the kernel's default decomposition (csrc/ops/gemm_stream.hip).
    rel: bit 0 = producer-side agent-scope release before the group barrier, bit 1 = each
    workgroup streams its K slice from a rotated starting chunk; None = STREAM_REL."""
    M, K = x.shape
    N = wp.shape[0] * 16
    code = STREAM_EPI[epi]
    NO = N // 2 if code == 1 else N
    if out is None:
        out = torch.empty(M, NO, dtype=x.dtype, device=x.device)
    if norm and ss_in is None:
        ss_in = row_sumsq(x)
    if _on_gpu(x):
        ws, cnt, err = stream_workspace(x.device)
        if not require_native().stream_gemm(out, x, wp, resid, ws, cnt, err, code, ss_in if norm else None, ss_out,
                                             ss_zero, float(eps), list(plan) if plan else [],
                                             rel=int(STREAM_REL if rel is None else rel),
                                             stamps=stamps):
            raise ValueError(f"stream_gemm does not handle M={M} N={N} K={K} epi={epi} plan={plan}")
        return out
    return mid_gemm(x, wp, epi, resid=resid, out=out, norm=norm, eps=eps, ss_in=ss_in, ss_out=ss_out,
                    ss_zero=ss_zero)


def stream_qkv_rope(x: torch.Tensor, wp: torch.Tensor, eps: float, q_out: torch.Tensor, k_cache, v_cache,
                    positions, slots, cos_sin, H: int, KV: int, ss_in: Optional[torch.Tensor] = None, plan=None,
                    rel: Optional[int] = None) -> torch.Tensor:
    """QKV projection for 16 < M <= 256 (RMSNorm folded, row statistics ss_in) with RoPE and the
    paged KV write in the epilogue (csrc/ops/gemm_stream.hip, EP_ROPEKV)."""
    if ss_in is None:
        ss_in = row_sumsq(x)
    if _on_gpu(x):
        ws, cnt, err = stream_workspace(x.device)
        if not require_native().stream_gemm(None, x, wp, None, ws, cnt, err, 4, ss_in, None, None, float(eps),
                                             list(plan) if plan else [], q_out, k_cache, v_cache, positions, slots,
                                             cos_sin, int(H), int(KV), int(STREAM_REL if rel is None else rel)):
            raise ValueError(f"stream_qkv_rope does not handle M={x.shape[0]} K={x.shape[1]} plan={plan}")
        return q_out
    return mid_qkv_rope(x, wp, eps, q_out, k_cache, v_cache, positions, slots, cos_sin, H, KV, ss_in=ss_in)


# ---------------------------------------------------------------------------
# Large-M projections (prefill-heavy steps) on the packed weights (csrc/ops/gemm_prefill.hip)

PREFILL_WS_FLOATS = 64 << 20  # 256 MB of split slabs per device (= gemm_prefill.hip kWsFloats)
_prefill_ws = {}


def prefill_workspace(device):
    """(slabs, tickets) for prefill_gemm / prefill_qkv_rope on `device`; allocate before
    hipGraph capture (the tickets start zeroed and every launch leaves them zeroed)."""
    key = str(device)
    if key not in _prefill_ws:
        _prefill_ws[key] = (empty_handoff(PREFILL_WS_FLOATS, torch.float32, device),
                            torch.zeros(16384, dtype=torch.int32, device=device))
    return _prefill_ws[key]


def prefill_gemm(x: torch.Tensor, wp: torch.Tensor, epi: str = "plain", resid: Optional[torch.Tensor] = None,
                 out: Optional[torch.Tensor] = None, norm: bool = False, eps: float = 1e-5, full: int = -1,
                 splits: int = 0, ss_in: Optional[torch.Tensor] = None, ss_out: Optional[torch.Tensor] = None,
                 ss_zero: Optional[torch.Tensor] = None, bn: int = 0, variant: int = -1) -> torch.Tensor:
    """y = epi(rownorm(x) @ W.T) for large M (256 x `bn` MFMA tiles, bn 128 / 256, 0 = the
    kernel's pick) with W packed by pack_decode_weight; same epilogues and row-statistics
    conventions as mid_gemm. `full` tiles run whole, the rest over `splits` K-slices (-1 / 0:
    the kernel's plan). `variant`: kernel family (3 ping-pong, 1 read-ahead / 3-stage;
    -1 = the process default)."""
    M, K = x.shape
    N = wp.shape[0] * 16
    code = MID_EPI[epi]
    NO = N // 2 if code == 1 else N
    if out is None:
        out = torch.empty(M, NO, dtype=x.dtype, device=x.device)
    if norm and ss_in is None:
        ss_in = row_sumsq(x)
    if _on_gpu(x):
        ws, cnt = prefill_workspace(x.device)
        if not _packed_module().prefill_gemm(out, x, wp, resid, ws, cnt, code, ss_in if norm else None, ss_out,
                                              ss_zero, float(eps), int(full), int(splits), int(bn), int(variant)):
            raise ValueError(f"prefill_gemm does not handle M={M} N={N} K={K} epi={epi} full={full} S={splits}")
        return out
    return mid_gemm(x, wp, epi, resid=resid, out=out, norm=norm, eps=eps, ss_in=ss_in, ss_out=ss_out,
                    ss_zero=ss_zero)


def prefill_qkv_rope(x: torch.Tensor, wp: torch.Tensor, eps: float, q_out: torch.Tensor, k_cache, v_cache,
                     positions, slots, cos_sin, H: int, KV: int, full: int = -1, splits: int = 0,
                     ss_in: Optional[torch.Tensor] = None, bn: int = 0, variant: int = -1) -> torch.Tensor:
    """Large-M QKV projection (RMSNorm folded, row statistics ss_in) with RoPE and the paged
    KV write in the epilogue (csrc/ops/gemm_prefill.hip EP_ROPEKV)."""
    if ss_in is None:
        ss_in = row_sumsq(x)
    if _on_gpu(x):
        ws, cnt = prefill_workspace(x.device)
        if not require_native().prefill_qkv_rope(x, wp, ss_in, float(eps), q_out, k_cache, v_cache, positions,
                                                  slots, cos_sin, int(H), int(KV), ws, cnt, int(full),
                                                  int(splits), int(bn), int(variant)):
            raise ValueError(f"prefill_qkv_rope does not handle M={x.shape[0]} K={x.shape[1]}")
        return q_out
    return mid_qkv_rope(x, wp, eps, q_out, k_cache, v_cache, positions, slots, cos_sin, H, KV, ss_in=ss_in)


def mid_qkv_rope(x: torch.Tensor, wp: torch.Tensor, eps: float, q_out: torch.Tensor, k_cache, v_cache, positions,
                 slots, cos_sin, H: int, KV: int, fm: int = 0, fn: int = 0, splits: int = 0,
                 ss_in: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Mid-size QKV projection with the RMSNorm folded in (norm weight pre-multiplied into
    the rope-packed weights; row statistics `ss_in`, computed here if absent), RoPE and the
    paged KV write in the epilogue: replaces rmsnorm + QKV GEMM + rope_cache on 49-512-token
    steps."""
    if ss_in is None:
        ss_in = row_sumsq(x)
    if _on_gpu(x):
        ws, cnt = mid_workspace(x.device)
        if not require_native().mid_qkv_rope(x, wp, ss_in, float(eps), q_out, k_cache, v_cache, positions, slots,
                                              cos_sin, int(H), int(KV), ws, cnt, int(fm), int(fn), int(splits)):
            raise ValueError(f"mid_qkv_rope does not handle M={x.shape[0]} K={x.shape[1]} fm={fm} fn={fn}")
        return q_out
    M, K = x.shape
    w = unpack_decode_qkv_rope(wp).float()
    qkv = (x.float() @ w.T) * torch.rsqrt(ss_in[:M].float().unsqueeze(-1) / K + eps)
    ref.rope_cache(q_out, k_cache, v_cache, qkv.to(x.dtype), positions, slots, cos_sin, H, KV)
    return q_out
