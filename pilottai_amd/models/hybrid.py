"""Sublayers of hybrid decoders: windowed attention with pooled keys, state-space (Mamba-2) layers,
gated feed-forwards and score-routed experts, on the engine's pages, state slots and packed projections.

Every class takes its sizes and constants from a spec, its weights by short names, and pads every
dimension with zero rows and columns to whole MFMA tiles at load, so any sizes run on the same kernels.
Each call takes the normed input h [T, >= width] and returns (y, partials, weights, bias): the
sublayer's output is bias + the weighted sum of a token's `partials` rows of y, which the residual
kernel takes directly.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, Optional, Tuple

import torch

from pilottai_amd import ops
from pilottai_amd.models.cache import StepMeta
from pilottai_amd.models.common import PackedLinear, expert_tile_rows
from pilottai_amd.ops.latent import pad_to

LINEAR_MAX = 3.0e38  # no clamp in the gated unit
SILU = (LINEAR_MAX, 1.0, 0.0, 0.0)  # (limit, alpha, bias, cubic) of ops.expert_gemm's gated unit
GELU_TANH = (LINEAR_MAX, 2.0 * (2.0 / 3.141592653589793) ** 0.5, 0.0, 0.044715)


@dataclass(frozen=True)
class PooledAttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_base: float
    rot_dims: int
    yarn: Optional[Tuple[float, float, float, float]] = None  # factor, original, fast, slow
    window: int = 0   # keys a position sees, itself included; 0: all before it
    pool: int = 0     # tokens of a pooled block before the window; 0: none
    sink: float = 1.0  # added to the softmax's denominator
    bias: bool = True  # of all four projections

    @property
    def group(self) -> int:
        return self.heads // self.kv_heads

    def angles(self, max_len: int) -> torch.Tensor:
        y = dict(zip(("factor", "original", "fast", "slow"), self.yarn)) if self.yarn else None
        return ops.angle_table(max_len, self.rot_dims, self.rot_base, y)

    def shapes(self, d: int) -> Dict[str, tuple]:
        n = {"q": (self.heads * self.dim, d), "k": (self.kv_heads * self.dim, d), "v": (self.kv_heads * self.vdim, d),
             "o": (d, self.heads * self.vdim)}
        return {**n, **({k + ".b": (s[0],) for k, s in n.items()} if self.bias else {})}


@dataclass(frozen=True)
class StateSpaceSpec:
    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int

    @property
    def padded(self) -> Tuple[int, int]:
        return pad_to(self.vdim, 16), pad_to(self.state, 32)

    @property
    def channels(self) -> int:  # of the convolution, padded
        vp, np_ = self.padded
        return self.heads * vp + 2 * self.groups * np_

    @property
    def ring_rows(self) -> int:
        return ops.conv_taps(self.conv) - 1 + ops.SCAN_MIN

    def shapes(self, d: int) -> Dict[str, tuple]:
        inner, bc = self.heads * self.vdim, 2 * self.groups * self.state
        h = (self.heads,)
        return {"in": (2 * inner + bc + self.heads, d), "conv": (inner + bc, self.conv), "conv.b": (inner + bc,),
                "dt_bias": h, "A_log": h, "D": h, "norm": (inner,), "o": (d, inner)}


@dataclass(frozen=True)
class DenseSpec:
    ff: int
    act: tuple = GELU_TANH

    def shapes(self, d: int) -> Dict[str, tuple]:
        return {"gate": (self.ff, d), "up": (self.ff, d), "down": (d, self.ff)}


@dataclass(frozen=True)
class ScoredExpertsSpec:
    experts: int
    top: int
    ff: int
    groups: int = 1   # equal groups of neighbouring experts
    keep: int = 1     # groups a token's experts may come from
    shared_ff: int = 0  # an expert of this width that runs for every token; 0: none
    act: tuple = SILU

    @property
    def always(self) -> int:  # the shared expert, in pieces of the routed experts' width
        return (self.shared_ff + self.ff - 1) // self.ff

    def shapes(self, d: int) -> Dict[str, tuple]:
        one = lambda f: {"gate": (f, d), "up": (f, d), "down": (d, f)}  # noqa: E731
        out = {"router": (self.experts, d)}
        for e in range(self.experts):
            out.update({f"e{e}.{k}": s for k, s in one(self.ff).items()})
        if self.shared_ff:
            out.update({f"shared.{k}": s for k, s in one(self.shared_ff).items()})
        return out


def _heads(w: torch.Tensor, n: int, size: int, padded: int) -> torch.Tensor:
    """[n * size, ...] -> [n * padded, ...], zeros behind every head."""
    out = w.new_zeros(n, padded, *w.shape[1:])
    out[:, :size] = w.reshape(n, size, *w.shape[1:])
    return out.reshape(n * padded, *w.shape[1:])


class PooledAttention:
    """Grouped-query attention over paged keys and values and their pooled blocks."""

    def __init__(self, spec: PooledAttentionSpec, t: Dict[str, torch.Tensor], dtype, device, cos_sin):
        m = self.spec = spec
        self.dtype, self.device, self.cos_sin = dtype, device, cos_sin
        H, G = m.heads, m.kv_heads
        self.dk, self.dv = ops.window_pad(m.dim, m.vdim)
        rows = lambda s: torch.cat([_heads(t["q" + s], H, m.dim, self.dk), _heads(t["k" + s], G, m.dim, self.dk),  # noqa: E731
                                    _heads(t["v" + s], G, m.vdim, self.dv)])
        self.qkv = PackedLinear(rows(""), dtype, device)
        self.bias = rows(".b").float().to(device).contiguous() if m.bias else None
        self.o = PackedLinear(_heads(t["o"].T.contiguous(), H, m.vdim, self.dv).T, dtype, device)
        self.o_bias = t["o.b"].float().to(device).contiguous() if m.bias else None

    def tensors(self):
        return [self.qkv.w, self.o.w]

    def __call__(self, h, meta: StepMeta, pages, part_o, part_ml, dec_tokens: int, tile_tokens: int, max_slots: int):
        m, T, H = self.spec, h.shape[0], self.spec.heads
        new = lambda *s: torch.empty(*s, dtype=self.dtype, device=self.device)  # noqa: E731
        kp, vp, pk, pv = pages
        x = self.qkv(h)
        q = new(T, H, self.dk)
        ops.paged_kv(x, self.bias, q, kp, vp, pk, pv, meta.positions, meta.slots, meta.q_start, meta.q_len, meta.ctx_len,
                     meta.block_table, self.cos_sin, m.pool if m.window else 0, num_seqs=meta.num_seqs)
        out = new(T, self.o.K)
        if self.o.K > H * self.dv:
            buf = new(T, H, self.dv)
            out[:, H * self.dv:] = 0
        else:
            buf = out.view(T, H, self.dv)
        ops.window_attention(buf, part_o, part_ml, q, kp, vp, pk, pv, meta.items, meta.n_items, meta.q_start, meta.q_len,
                             meta.ctx_len, meta.block_table, m.scale, m.window, m.pool if m.window else 0, m.sink,
                             dec_tokens, tile_tokens, max_slots, num_seqs=meta.num_seqs)
        if self.o.K > H * self.dv:
            out[:, :H * self.dv] = buf.view(T, -1)
        return self.o(out), 1, None, self.o_bias


class StateSpace:
    """Mamba-2: projection, causal convolution, recurrence, gated grouped norm, output projection."""

    def __init__(self, spec: StateSpaceSpec, t: Dict[str, torch.Tensor], eps: float, dtype, device):
        m = self.spec = spec
        self.eps, self.dtype, self.device = eps, dtype, device
        H, V, N, G = m.heads, m.vdim, m.state, m.groups
        inner, (vp, np_) = H * V, m.padded
        self.vp, self.inner = vp, H * vp

        def channels(w):  # x | B | C
            return torch.cat([_heads(w[:inner], H, V, vp), _heads(w[inner:inner + G * N], G, N, np_),
                              _heads(w[inner + G * N:], G, N, np_)])
        z, xbc, dt = torch.split(t["in"], [inner, inner + 2 * G * N, H])
        self.w_in = PackedLinear(torch.cat([_heads(z, H, V, vp), channels(xbc), dt]), dtype, device)
        f32 = lambda x: x.float().to(device).contiguous()  # noqa: E731
        conv = t["conv"].float()
        conv = torch.cat([conv.new_zeros(conv.shape[0], ops.conv_taps(m.conv) - m.conv), conv], 1)
        self.conv_w, self.conv_b = f32(channels(conv).T), f32(channels(t["conv.b"]))
        self.dt_bias, self.a, self.d = f32(t["dt_bias"]), f32(torch.exp(t["A_log"].float())), f32(t["D"])
        self.w_norm = f32(t["norm"])
        self.o = PackedLinear(_heads(t["o"].T.contiguous(), H, V, vp).T, dtype, device)

    def tensors(self):
        return [self.w_in.w, self.o.w]

    def __call__(self, h, meta: StepMeta, cache):
        m = self.spec
        state, ring = cache
        x = self.w_in(h)
        y = torch.empty(h.shape[0], self.o.K, dtype=self.dtype, device=self.device)
        ops.state_scan(x, y, state, ring, self.conv_w, self.conv_b, self.dt_bias, self.a, self.d, meta.q_start, meta.q_len,
                       meta.ctx_len, meta.state_slot, meta.scan_first, meta.scan_items, meta.n_scan, m.groups,
                       num_seqs=meta.num_seqs)
        ops.gated_norm(y, x, self.w_norm, meta.slots, m.heads, m.vdim, self.vp, m.norm_groups, self.eps)
        return self.o(y), 1, None, None


def _pack_gate_up(gate, up, fp: int, dk: int, dtype, device):
    g = torch.zeros(2, 1, fp, dk, dtype=dtype, device=device)
    f, d = gate.shape
    g[0, 0, :f, :d], g[1, 0, :f, :d] = gate.to(device), up.to(device)
    return ops.pack_groups(ops.interleave_gate_up(g[0], g[1]), dtype)


class GatedMLP:
    """down(act(gate h) * up h): the gate and up rows interleaved in one grouped projection of one group."""

    # 16-row tiles (each streams the weights) up to this many rows, by weights that passes find in the caches again
    ROWS_16, ROWS_16_LARGE, LARGE = 80, 40, 1 << 26

    def __init__(self, spec: DenseSpec, t: Dict[str, torch.Tensor], width: int, dtype, device):
        self.spec, self.dtype, self.device = spec, dtype, device
        self.dk = pad_to(width, 64)
        self.down = PackedLinear(t["down"], dtype, device)
        self.fp = self.down.K
        self.w13 = _pack_gate_up(t["gate"], t["up"], self.fp, self.dk, dtype, device)
        self._tiles: Dict[int, tuple] = {}

    def tensors(self):
        return [self.w13, self.down.w]

    def __call__(self, h, meta: StepMeta):
        T = h.shape[0]
        if T not in self._tiles:  # (before graph capture: the capture's warm-up runs come first)
            few = self.ROWS_16 if self.w13.numel() <= self.LARGE else self.ROWS_16_LARGE
            tm = expert_tile_rows(T, self.dtype, self.dk, few, few)
            tiles = torch.tensor([[0, i, min(tm, T - i), 0] for i in range(0, T, tm)], dtype=torch.int32)
            self._tiles[T] = (tiles.to(self.device), torch.tensor([len(tiles)], dtype=torch.int32, device=self.device),
                              torch.arange(T, dtype=torch.int32, device=self.device), tm)
        tiles, n, order, tm = self._tiles[T]
        act = torch.empty(T, self.fp, dtype=self.dtype, device=self.device)
        ops.expert_gemm(h, self.w13, act, tiles, n, order, T, x_div=0, out_order=False, tm=tm, glu=self.spec.act)
        return self.down(act), 1, None, None


class ScoredExperts:
    """Experts chosen by the scores of a router, and a shared expert whose pieces are further experts that
    every token uses; one partial output per (token, expert) with its weight."""

    ROWS_64, ROWS_256 = 32, 96  # average rows per expert above which they go in tiles of 64 / 256

    def __init__(self, spec: ScoredExpertsSpec, t: Dict[str, torch.Tensor], width: int, dtype, device):
        s = self.spec = spec
        self.dtype, self.device = dtype, device
        f, dk, dn = s.ff, pad_to(width, 64), pad_to(width, 128)
        self.fp, self.dk, self.dn = pad_to(f, 64), dk, dn
        w13, w2 = [], []

        def add(gate, up, down):
            w13.append(_pack_gate_up(gate, up, self.fp, dk, dtype, device))
            w = torch.zeros(1, dn, self.fp, dtype=dtype, device=device)
            w[0, :width, :down.shape[1]] = down.to(device)
            w2.append(ops.pack_groups(w, dtype))
        for e in range(s.experts):
            add(t[f"e{e}.gate"], t[f"e{e}.up"], t[f"e{e}.down"])
        for i in range(s.always):
            a, b = i * f, min((i + 1) * f, s.shared_ff)
            add(t["shared.gate"][a:b], t["shared.up"][a:b], t["shared.down"][:, a:b])
        self.w13, self.w2 = torch.cat(w13), torch.cat(w2)
        r = torch.zeros(1, pad_to(s.experts, 16), dk, dtype=dtype, device=device)
        r[0, :s.experts, :width] = t["router"].to(device)
        self.router = ops.pack_groups(r, dtype)

    def tensors(self):
        return [self.w13, self.w2, self.router]

    def __call__(self, h, meta: StepMeta):
        s, T, dev = self.spec, h.shape[0], self.device
        E, K = s.experts + s.always, s.top + s.always
        tm = expert_tile_rows(T * s.top / s.experts, self.dtype, min(self.fp, self.dk), self.ROWS_64, self.ROWS_256)
        rows = T * K
        ints = lambda *n: torch.empty(*n, dtype=torch.int32, device=dev)  # noqa: E731
        weights = torch.empty(T, K, dtype=torch.float32, device=dev)
        choice, rank, order, tiles, n_tiles = ints(rows), ints(rows), ints(rows), ints(rows // tm + min(E, rows), 4), ints(1)
        counts = torch.zeros(E, dtype=torch.int32, device=dev) if T > 16 else ints(E)  # (small steps: unused)
        ops.score_route(h, self.router, meta.slots, weights, choice, rank, counts, order, tiles, n_tiles, s.experts, s.top,
                        s.groups, s.keep, s.always, tm)
        act = torch.empty(rows, self.fp, dtype=self.dtype, device=dev)
        ops.expert_gemm(h, self.w13, act, tiles, n_tiles, order, rows, x_div=K, out_order=False, tm=tm, glu=s.act)
        y = torch.empty(rows, self.dn, dtype=self.dtype, device=dev)
        ops.expert_gemm(act, self.w2, y, tiles, n_tiles, order, rows, x_div=0, out_order=True, tm=tm)
        return y, K, weights, None
