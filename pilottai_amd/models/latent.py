"""Latent attention over the paged latent cache, queries absorbed into the latent space: one cached row per token for
all heads, [latent | rotated key part].

    c = norm(W_dkv h),  page row = [c | rot(k_r)]         (or the rows of an earlier layer, `kv_from`)
    [q_n | q_r] = W_uq norm(W_dq h), or W_q h;   q~_h = [W_uk,h^T q_n,h | rot(q_r,h)]
    p_h = softmax(scale * q~_h . row(j)),  0 <= i - j < window
    o_h = W_uv,h sum_j p_h c_j, times sigmoid(W_g h) if gated

LatentAttention is a mixer of models/hybrid.py MixerBlock, which holds its first and its output matrix.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, Optional

import torch

from pilottai_amd import ops
from pilottai_amd.models.cache import StepMeta
from pilottai_amd.models.common import PackedLinear, pad_heads
from pilottai_amd.ops.latent import latent_pad, pad_to


@dataclass(frozen=True)
class LatentAttentionSpec:
    heads: int
    dim: int          # unrotated query / key dimensions per head
    vdim: int
    kv_rank: int
    scale: float
    q_rank: int = 0   # queries through a latent of this size; 0: straight from the input
    rot_dim: int = 0  # rotated dimensions per head (one key part shared by all heads); 0: none
    rot_base: float = 1.0
    rot_dims: int = 0  # rotated dimensions of rot_dim
    rot_pairs: bool = False  # neighbours turn together; else the two halves
    window: int = 0   # keys a position sees, itself included; 0: all before it
    gate: bool = False  # the heads' outputs times sigmoid(W_g h)
    kv_from: Optional[int] = None  # the layer whose cached latents these heads read

    def __post_init__(self):
        if self.rot_dims > self.rot_dim or self.rot_dims % 2:
            raise ValueError(f"{self.rot_dims} rotated of {self.rot_dim} dimensions")
        if self.scale <= 0 or self.kv_from is not None and (self.rot_dim or self.q_rank):
            raise ValueError("unsupported latent attention")

    # every head reads the same row: one key head for all of them
    kv_heads = maps = 1
    pool = 0

    @property
    def group(self) -> int:
        return self.heads

    @property
    def max_keys(self) -> int:
        return self.window

    @property
    def out_width(self) -> int:  # of a head's output before W_uv
        return latent_pad(self.kv_rank)

    @property
    def rotation(self) -> tuple:
        return self.rot_dims, self.rot_base

    def angles(self, max_len: int) -> torch.Tensor:
        return ops.angle_table(max_len, self.rot_dims, self.rot_base)

    def shapes(self, d: int) -> Dict[str, tuple]:
        H, n = self.heads, self.dim + self.rot_dim
        out = {"dq": (self.q_rank, d), "dq.norm": (self.q_rank,), "uq": (H * n, self.q_rank)} if self.q_rank else {"q": (H * n, d)}
        if self.kv_from is None:
            out.update({"dkv": (self.kv_rank + self.rot_dim, d), "dkv.norm": (self.kv_rank,)})
        out.update({"uk": (H * self.dim, self.kv_rank), "uv": (H * self.vdim, self.kv_rank), "o": (d, H * self.vdim)})
        if self.gate:
            out["g"] = (H * self.vdim, d)
        return out


class LatentAttention:
    """Projection rows [query latent or queries | latent | rotated key part | gate]. `source`: the mixer of the layer
    that kv_from names."""

    def __init__(self, spec: LatentAttentionSpec, t: Dict[str, torch.Tensor], eps: float, dtype, device, cos_sin=None,
                 source: Optional["LatentAttention"] = None):
        m = self.spec = spec
        self.eps, self.dtype, self.device, self.cos_sin = eps, dtype, device, cos_sin
        H, n, r, vd, R = m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank
        self.np, self.rp, self.vp = pad_to(n, 32), pad_to(r, 32), pad_to(vd, 16)
        self.Rp = latent_pad(R)
        self.D = self.Rp + self.rp if source is None else source.D
        f32 = lambda x: x.float().to(device).contiguous()  # noqa: E731

        def turned(w):  # the rotation's pairs as halves, [.., r, k]
            if not m.rot_pairs:
                return w
            a = w[..., :m.rot_dims, :]
            return torch.cat([a[..., 0::2, :], a[..., 1::2, :], w[..., m.rot_dims:, :]], -2)
        q = t["uq" if m.q_rank else "q"].view(H, n + r, -1)
        q = torch.cat([pad_heads(q[:, :n], self.np), pad_heads(turned(q[:, n:]), self.rp)], 1).reshape(H * (self.np + self.rp), -1)
        self.uq = PackedLinear(q, dtype, device) if m.q_rank else None
        rows = [t["dq"] if m.q_rank else q]
        self.c_col = 0 if m.q_rank else q.shape[0]  # of [query latent |] latent | rotated key part
        self.w_q = f32(t["dq.norm"]) if m.q_rank else None
        self.w_c = None
        if source is None:
            rows += [t["dkv"][:R], turned(t["dkv"][R:])]
            self.w_c = f32(t["dkv.norm"])
        if m.gate:
            n_rows = sum(w.shape[0] for w in rows)
            self.g_col = pad_to(n_rows, 16)
            rows += [rows[0].new_zeros(self.g_col - n_rows, rows[0].shape[1]),
                     pad_heads(t["g"].view(H, vd, -1), self.vp).reshape(H * self.vp, -1)]
        self.rows = torch.cat(rows)
        uk = torch.zeros(H, self.Rp, self.np, dtype=dtype, device=device)
        uk[:, :R, :n] = t["uk"].to(device).view(H, n, R).transpose(1, 2)
        self.uk = ops.pack_groups(uk, dtype)
        uv = torch.zeros(H, self.vp, self.Rp, dtype=dtype, device=device)
        uv[:, :vd, :R] = t["uv"].to(device).view(H, vd, R)
        self.uv = ops.pack_groups(uv, dtype)
        self.width, self.out_bias = H * self.vp, None
        self.w_out = pad_heads(t["o"].T.reshape(H, vd, -1), self.vp).reshape(self.width, -1).T

    def tensors(self):
        return ([self.uq.w] if self.uq else []) + [self.uk, self.uv]

    def cache_kind(self) -> tuple:
        return ("latent", self.D) if self.spec.kv_from is None else ("same", self.spec.kv_from)

    def __call__(self, x, out, meta: StepMeta, cache, room):
        m, T, H = self.spec, x.shape[0], self.spec.heads
        pages, = cache
        new = lambda *s: torch.empty(*s, dtype=self.dtype, device=self.device)  # noqa: E731
        cq = new(T, self.uq.K) if self.uq else None
        if m.kv_from is None:
            ops.latent_cache(x[:, self.c_col:], m.q_rank, m.kv_rank, m.rot_dim, self.w_q, self.w_c, cq, pages, self.Rp,
                             meta.positions, meta.slots, self.cos_sin, self.eps)
        q = self.uq(cq) if self.uq else x
        qa = new(T, H, self.D)
        if self.D > self.Rp + self.rp:  # (another layer's rows have a rotated part, which these queries leave out)
            qa.zero_()
        ops.head_gemm(q, self.np + self.rp, self.uk, qa.view(T, -1), self.D,
                      rot=(meta.positions, self.cos_sin, self.np, m.rot_dim, self.rp) if m.rot_dim else None)
        oc = new(T, H, self.Rp)
        ops.latent_attention(oc, room.part_o, room.part_ml, qa, pages, meta.items, meta.n_items, meta.q_start,
                             meta.q_len, meta.ctx_len, meta.block_table, m.scale, m.window, room.dec_tokens, room.tile_tokens,
                             num_seqs=meta.num_seqs)
        ops.head_gemm(oc.view(T, -1), self.Rp, self.uv, out, self.vp, gate=x[:, self.g_col:] if m.gate else None)
