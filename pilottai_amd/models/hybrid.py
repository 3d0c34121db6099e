"""Sublayers of hybrid decoders: attention over paged keys and values, recurrent layers (Mamba-2, matrix
memory, gated linear attention), dense feed-forwards and score-routed experts, on the engine's pages, state slots and packed
projections; and what the models made of them have in common.

Every class takes its sizes and constants from a spec, its weights by short names, and pads every
dimension with zero rows and columns to whole MFMA tiles at load, so any sizes run on the same kernels.

A mixer (PagedAttention, StateSpace, MatrixMemory, LinearAttention; models/latent.py LatentAttention) reads its columns of a projection of the normed input and writes
columns that an output matrix takes: `rows` and `w_out` are its parts of those two matrices. A MixerBlock holds
them for one mixer or several side by side, and, where a feed-forward reads the same input, for that one's
second matrix too: one projection, one output product. Blocks and feed-forwards return (y, partials, weights,
bias): their output is bias + the weighted sum of a token's `partials` rows of y, which the residual kernel
takes directly.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, NamedTuple, Optional, Sequence, Tuple

import torch

from pilottai_amd import ops
from pilottai_amd.models.cache import HybridCache, StepMeta
from pilottai_amd.models.common import PackedLinear, checkpoint_reader, expert_tile_rows
from pilottai_amd.ops.latent import pad_to
from pilottai_amd.parallel.comm import TPGroup

LINEAR_MAX = 3.0e38  # no clamp in the gated unit
SILU = (LINEAR_MAX, 1.0, 0.0, 0.0)  # (limit, alpha, bias, cubic) of ops.expert_gemm's gated unit
GELU_TANH = (LINEAR_MAX, 2.0 * (2.0 / 3.141592653589793) ** 0.5, 0.0, 0.044715)
MAX_NORMED = 512  # widest head that paged_kv norms


@dataclass(frozen=True)
class AttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_base: float = 1.0
    rot_dims: int = 0  # 0: no rotation
    yarn: Optional[Tuple[float, float, float, float]] = None  # factor, original, fast, slow
    slow_waves: Optional[Tuple[float, float, float, float]] = None  # factor, low, high, original
    window: int = 0   # keys a position sees, itself included; 0: all before it
    pool: int = 0     # tokens of a pooled block before the window; 0: none
    keep: int = 0     # first tokens that stay visible behind the window
    chunk: int = 0    # a position sees its own chunk of so many positions; 0: no chunks
    slopes: Optional[Tuple[float, ...]] = None  # per head: slope * distance is taken off the score
    cap: float = 0.0  # scores are cap tanh(s / cap); 0: none
    sink: float = 0.0  # a constant added to the softmax's denominator
    learned_sink: bool = False  # exp(tensor 'sink') is added, a number per head
    bias: bool = False  # of all four projections
    qk_norm: bool = False  # RMS norm of every query and key head, before the rotation
    v_norm: bool = False   # of every value head, without a weight
    keys_as_values: bool = False  # no value projection: the keys as projected
    gate: bool = False  # the heads' outputs times sigmoid(W_g h)
    diff: Optional[float] = None  # two maps per head over the same values, the second taken off the first

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} heads do not divide over {self.kv_heads} key/value heads")
        if self.rot_dims > self.dim or self.rot_dims % 2:
            raise ValueError(f"{self.rot_dims} rotated of {self.dim} dimensions")
        if self.keys_as_values and self.dim != self.vdim:
            raise ValueError(f"keys of {self.dim} as values of {self.vdim}")
        if (self.chunk or self.keep) and self.pool or self.chunk and self.window or self.keep and not self.window:
            raise ValueError("kept tokens go with a window; chunks, and pooled blocks, with neither")
        if (self.qk_norm and self.dim > MAX_NORMED) or \
                ((self.v_norm or self.diff is not None) and self.vdim > MAX_NORMED):
            raise ValueError(f"normed heads of more than {MAX_NORMED} dimensions")
        if self.scale <= 0 or (self.diff is not None and (self.bias or not self.gate or self.pool or self.keys_as_values)):
            raise ValueError("unsupported attention")

    @property
    def maps(self) -> int:
        return 1 if self.diff is None else 2

    @property
    def group(self) -> int:
        return self.heads // self.kv_heads

    @property
    def max_keys(self) -> int:
        """Tokens a position sees at most (0: no limit)."""
        return self.chunk or (self.window + self.keep if self.window else 0)

    @property
    def rotation(self) -> tuple:
        return self.rot_dims, self.rot_base, self.yarn, self.slow_waves

    @property
    def out_width(self) -> int:
        return ops.window_pad(self.dim, self.vdim)[1]

    def angles(self, max_len: int) -> torch.Tensor:
        named = lambda v, k: dict(zip(k, v)) if v else None  # noqa: E731
        return ops.angle_table(max_len, self.rot_dims, self.rot_base, named(self.yarn, ("factor", "original", "fast", "slow")),
                               named(self.slow_waves, ("factor", "low", "high", "original")))

    def shapes(self, d: int) -> Dict[str, tuple]:
        n = {"q": (self.heads * self.maps * self.dim, d), "k": (self.kv_heads * self.maps * self.dim, d)}
        if not self.keys_as_values:
            n["v"] = (self.kv_heads * self.vdim, d)
        n["o"] = (d, self.heads * self.vdim)
        out = {**n, **({k + ".b": (s[0],) for k, s in n.items()} if self.bias else {})}
        if self.qk_norm:
            out.update({"q.norm": (self.dim,), "k.norm": (self.dim,)})
        if self.learned_sink:
            out["sink"] = (self.heads,)
        if self.gate:
            out["g"] = (self.heads * self.vdim, d)
        if self.diff is not None:
            out.update({k: (self.dim,) for k in ("lq1", "lk1", "lq2", "lk2")})
        return out


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
class MatrixMemorySpec:
    heads: int
    dim: int
    vdim: int
    cap: float  # of the gates before their exponentials

    @property
    def padded(self) -> Tuple[int, int, int]:
        """Widths of a key, of a value in the projection, and of a value and the keys' sum in the state."""
        return pad_to(self.dim, 32), pad_to(self.vdim, 16), pad_to(self.vdim + 1, 16)

    def shapes(self, d: int) -> Dict[str, tuple]:
        H, N, V = self.heads, self.heads * self.dim, self.heads * self.vdim
        return {"q": (N, d), "k": (N, d), "v": (V, d), "g": (V, d), "o": (d, V), "norm": (V,),
                "i": (H, d), "i.b": (H,), "f": (H, d), "f.b": (H,)}


@dataclass(frozen=True)
class LinearAttentionSpec:
    heads: int
    dim: int
    vdim: int
    tau: float  # decays are sigmoid(z)^(1 / tau)
    rank: int = 16  # of the map from the input to z

    def __post_init__(self):
        if self.tau <= 0:
            raise ValueError(f"decays with tau {self.tau}")

    @property
    def padded(self) -> Tuple[int, int, int]:
        """Widths of a key, a value and the decays' low-rank input."""
        return pad_to(self.dim, 32), pad_to(self.vdim, 16), pad_to(self.rank, 32)

    def shapes(self, d: int) -> Dict[str, tuple]:
        N, V = self.heads * self.dim, self.heads * self.vdim
        return {"q": (N, d), "k": (N, d), "v": (V, d), "g": (V, d), "o": (d, V), "norm": (self.vdim,), "a1": (self.rank, d),
                "a2": (N, self.rank), "a2.b": (N,)}


@dataclass(frozen=True)
class PolySpec:
    """A feed-forward without a gate whose activation is the polynomial norm of the token's vector."""
    ff: int

    def shapes(self, d: int) -> Dict[str, tuple]:
        return {"up": (self.ff, d), "down": (d, self.ff), "act": (4,)}


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
    act: Optional[tuple] = SILU  # of gated experts; None: no gate, the square of relu
    softmax: bool = False  # scores over all experts; else a sigmoid each
    correction: bool = False  # the choice is by score + tensor 'correction'
    share: bool = False  # weights: the chosen scores divided by their sum
    scale: float = 1.0   # of the weights
    weigh_input: bool = False  # an expert's weight multiplies its input; else its output

    def __post_init__(self):
        if self.experts % self.groups or not 1 <= self.keep <= self.groups or \
                not 1 <= self.top <= self.keep * (self.experts // self.groups):
            raise ValueError(f"{self.top} of {self.experts} experts from {self.keep} of {self.groups} groups")
        if self.weigh_input and self.act is None:
            raise ValueError("weights on the input of experts without a gate")

    @property
    def always(self) -> int:  # the shared expert, in pieces of the routed experts' width
        return (self.shared_ff + self.ff - 1) // self.ff

    def shapes(self, d: int) -> Dict[str, tuple]:
        one = lambda f: {**({"gate": (f, d)} if self.act else {}), "up": (f, d), "down": (d, f)}  # noqa: E731
        out = {"router": (self.experts, d), **({"correction": (self.experts,)} if self.correction else {})}
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


class SideStreams:
    """Streams for branches of a step that do not depend on each other. They are used while a graph is captured, whose
    replays then run the branches together; an eager step runs them one after the other. A branch's tensors are
    its stream's: the next step of that stream waits for whoever has read them."""

    def __init__(self, device, count: int):
        self.streams = [torch.cuda.Stream(device) for _ in range(count)] if device.type == "cuda" else []

    def run(self, first, *others, at: int = 0):
        """Results of first() and others(), the latter on the streams from number `at` on."""
        if not self.streams or not torch.cuda.is_current_stream_capturing():
            return [f() for f in (first, *others)]
        main, out = torch.cuda.current_stream(), []
        used = self.streams[at:at + len(others)]
        for s, f in zip(used, others):
            s.wait_stream(main)
            with torch.cuda.stream(s):
                out.append(f())
        out.insert(0, first())
        for s in used:
            main.wait_stream(s)
        return out


class AttentionRoom(NamedTuple):
    """What the engine's attention work items need: partial results and the tokens of an item."""
    part_o: torch.Tensor
    part_ml: torch.Tensor
    dec_tokens: int
    tile_tokens: int
    max_slots: int


class PagedAttention:
    """Grouped-query attention over paged keys and values; differential attention has two key heads per value
    head, in the order (KV head, map, query head of the group)."""

    def __init__(self, spec: AttentionSpec, t: Dict[str, torch.Tensor], dtype, device, cos_sin=None, eps: float = 0.0,
                 gain: float = 1.0):
        m = self.spec = spec
        self.dtype, self.device, self.cos_sin, self.eps, self.gain = dtype, device, cos_sin, eps, gain
        H, G, M = m.heads, m.kv_heads, m.maps
        self.dk, self.dv = ops.window_pad(m.dim, m.vdim)
        self.nq, self.nk, self.width = H * M, G * M, H * self.dv
        f32 = lambda x: x.float().to(device).contiguous()  # noqa: E731

        def rows(s):
            q = t["q" + s].reshape(G, m.group, M, m.dim, -1).transpose(1, 2).reshape(H * M * m.dim, *t["q" + s].shape[1:])
            parts = [_heads(q, H * M, m.dim, self.dk), _heads(t["k" + s], G * M, m.dim, self.dk)]
            return torch.cat(parts + ([] if m.keys_as_values else [_heads(t["v" + s], G, m.vdim, self.dv)]))
        self.rows = rows("")
        self.bias = f32(rows(".b")) if m.bias else None
        self.v_col = self.nq * self.dk if m.keys_as_values else -1
        self.g_col = self.rows.shape[0]
        if m.gate:
            self.rows = torch.cat([self.rows, _heads(t["g"], H, m.vdim, self.dv)])
        self.w_out = _heads(t["o"].T.contiguous(), H, m.vdim, self.dv).T
        self.out_bias = f32(t["o.b"]) if m.bias else None
        pad = lambda w: torch.cat([f32(w), torch.zeros(self.dk - m.dim, device=device)])  # noqa: E731
        self.q_norm, self.k_norm = (pad(t["q.norm"]), pad(t["k.norm"])) if m.qk_norm else (None, None)
        self.slopes = torch.tensor(m.slopes, dtype=torch.float32, device=device) if m.slopes else None
        self.sink = f32(t["sink"]) if m.learned_sink else \
            torch.full((H,), float(m.sink), device=device).log() if m.sink > 0 else None
        if m.diff is not None:
            dot = lambda i: float((t[f"lq{i}"].double() * t[f"lk{i}"].double()).sum().exp())  # noqa: E731
            self.lam = dot(1) - dot(2) + m.diff

    def cache_kind(self) -> tuple:
        m = self.spec
        return ("attention", self.nk, self.dk, self.dv, ops.pooled_per_page(m.pool) if m.pool and m.window else 0, m.kv_heads)

    def __call__(self, x, out, meta: StepMeta, cache, room: AttentionRoom):
        m, T = self.spec, x.shape[0]
        kp, vp, pk, pv = cache
        pool = m.pool if m.window else 0
        q = torch.empty(T, self.nq, self.dk, dtype=self.dtype, device=self.device)
        ops.paged_kv(x, self.bias, q, kp, vp, pk, pv, meta.positions, meta.slots, meta.q_start, meta.q_len, meta.ctx_len,
                     meta.block_table, self.cos_sin, pool, num_seqs=meta.num_seqs, v_col=self.v_col, q_norm=self.q_norm,
                     k_norm=self.k_norm, norm_v=m.v_norm, dim=m.dim, vdim=m.vdim, eps=self.eps)
        o = out[:, :self.width].view(T, m.heads, self.dv)
        gate = x[:, self.g_col:self.g_col + self.width] if m.gate else None
        # (the maps' outputs stay in fp32: their difference is small against them)
        a = o if m.diff is None else torch.empty(T, self.nq, self.dv, dtype=torch.float32, device=self.device)
        ops.window_attention(a, room.part_o, room.part_ml, q, kp, vp, pk, pv, meta.items, meta.n_items, meta.q_start, meta.q_len,
                             meta.ctx_len, meta.block_table, m.scale, m.window, pool, self.sink, room.dec_tokens, room.tile_tokens,
                             room.max_slots, num_seqs=meta.num_seqs, keep=m.keep, chunk=m.chunk, slopes=self.slopes, cap=m.cap,
                             gate=gate if m.diff is None else None, gain=self.gain if m.diff is None else 1.0)
        if m.diff is not None:
            ops.head_difference(a, o, gate, m.kv_heads, self.lam, (1.0 - m.diff) * self.gain, m.vdim, self.eps)


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
        self.rows = torch.cat([_heads(z, H, V, vp), channels(xbc), dt])
        f32 = lambda x: x.float().to(device).contiguous()  # noqa: E731
        conv = t["conv"].float()
        conv = torch.cat([conv.new_zeros(conv.shape[0], ops.conv_taps(m.conv) - m.conv), conv], 1)
        self.conv_w, self.conv_b = f32(channels(conv).T), f32(channels(t["conv.b"]))
        self.dt_bias, self.a, self.d = f32(t["dt_bias"]), f32(torch.exp(t["A_log"].float())), f32(t["D"])
        self.w_norm = f32(t["norm"])
        self.w_out, self.out_bias, self.width = _heads(t["o"].T.contiguous(), H, V, vp).T, None, H * vp

    def cache_kind(self) -> tuple:
        m = self.spec
        return ("state", m.heads, *m.padded, m.ring_rows, m.channels)

    def __call__(self, x, out, meta: StepMeta, cache, room):
        m = self.spec
        state, ring = cache
        ops.state_scan(x, out, state, ring, self.conv_w, self.conv_b, self.dt_bias, self.a, self.d, meta.q_start, meta.q_len,
                       meta.ctx_len, meta.state_slot, meta.scan_first, meta.scan_items, meta.n_scan, m.groups,
                       num_seqs=meta.num_seqs)
        ops.gated_norm(out, x, self.w_norm, meta.slots, m.heads, m.vdim, self.vp, m.norm_groups, self.eps)


class MatrixMemory:
    """mLSTM: an outer-product memory per head with exponential gates held by a running maximum, its output divided
    by the memory's weight, normed per head and gated. Projection rows [q | k | v | gate | i | f]."""

    def __init__(self, spec: MatrixMemorySpec, t: Dict[str, torch.Tensor], eps: float, dtype, device, gain: float = 1.0):
        m = self.spec = spec
        self.eps, self.dtype, self.device = eps, dtype, device
        H, (np_, vin, _) = m.heads, m.padded
        self.rows = torch.cat([_heads(t["q"], H, m.dim, np_), _heads(t["k"], H, m.dim, np_), _heads(t["v"], H, m.vdim, vin),
                               _heads(t["g"], H, m.vdim, vin), t["i"], t["f"]])
        self.g_col = 2 * H * np_ + H * vin
        self.cols = (0, H * np_, 2 * H * np_, self.g_col + H * vin, vin)
        f32 = lambda x: x.float().to(device).contiguous()  # noqa: E731
        self.i_bias, self.f_bias, self.w_norm = f32(t["i.b"]), f32(t["f.b"]), f32(t["norm"].float() * gain)
        self.w_out, self.out_bias, self.width = _heads(t["o"].T.contiguous(), H, m.vdim, vin).T, None, H * vin

    def cache_kind(self) -> tuple:
        np_, _, vs = self.spec.padded
        return ("memory", self.spec.heads, vs, np_)

    def __call__(self, x, out, meta: StepMeta, cache, room):
        m, T = self.spec, x.shape[0]
        state, top = cache
        div = torch.empty(T, m.heads, dtype=torch.float32, device=self.device)
        ops.matrix_memory(x, out, div, state, top, self.i_bias, self.f_bias, meta.q_start, meta.q_len, meta.ctx_len,
                          meta.state_slot, meta.scan_items, meta.n_scan, self.cols, m.vdim, m.cap, m.dim ** -0.5,
                          num_seqs=meta.num_seqs)
        ops.gated_norm(out, x[:, self.g_col:], self.w_norm, meta.slots, m.heads, m.vdim, self.cols[4], m.heads, self.eps,
                       div=div, after="sigmoid")


class LinearAttention:
    """Gated linear attention: an outer-product state per head whose key channels decay each by itself, its output normed
    per head and gated. Projection rows [q | k | v | gate | low-rank inputs of the decays]."""

    def __init__(self, spec: LinearAttentionSpec, t: Dict[str, torch.Tensor], eps: float, dtype, device):
        m = self.spec = spec
        self.eps, self.dtype, self.device = eps, dtype, device
        H, (np_, vp, rp) = m.heads, m.padded
        self.rows = torch.cat([_heads(t["q"], H, m.dim, np_), _heads(t["k"], H, m.dim, np_), _heads(t["v"], H, m.vdim, vp),
                               _heads(t["g"], H, m.vdim, vp), t["a1"], t["a1"].new_zeros(rp - m.rank, t["a1"].shape[1])])
        self.g_col = 2 * H * np_ + H * vp
        self.cols = (0, H * np_, 2 * H * np_, self.g_col + H * vp)
        self.a2 = torch.zeros(H * np_, rp, dtype=dtype, device=device)
        self.a2[:, :m.rank] = _heads(t["a2"], H, m.dim, np_).to(device)
        f32 = lambda x: x.float().to(device).contiguous()  # noqa: E731
        self.bias, self.w_norm = f32(_heads(t["a2.b"], H, m.dim, np_)), f32(t["norm"].repeat(H))
        self.w_out, self.out_bias, self.width = _heads(t["o"].T.contiguous(), H, m.vdim, vp).T, None, H * vp

    def tensors(self):
        return [self.a2]

    def cache_kind(self) -> tuple:
        np_, vp, _ = self.spec.padded
        return ("linear", self.spec.heads, vp, np_)

    def __call__(self, x, out, meta: StepMeta, cache, room):
        m = self.spec
        state, = cache
        ops.linear_attention(x, out, state, self.a2, self.bias, meta.q_start, meta.q_len, meta.ctx_len, meta.state_slot,
                             meta.scan_items, meta.n_scan, self.cols, m.dim ** -0.5, 1.0 / m.tau, num_seqs=meta.num_seqs)
        ops.gated_norm(out, x[:, self.g_col:], self.w_norm, meta.slots, m.heads, m.vdim, m.padded[1], m.heads, self.eps,
                       after="silu")


class MixerBlock:
    """Mixers side by side on one projection and one output matrix. `mlp`: a GatedMLP that reads the same input and
    whose second matrix is part of the output matrix."""

    def __init__(self, mixers: Sequence, dtype, device, mlp: Optional["GatedMLP"] = None):
        self.mixers, self.mlp, self.dtype, self.device = list(mixers), mlp, dtype, device
        self.at_in: List[int] = []
        self.at_out: List[int] = []
        rows, outs, n = [], [], 0
        for m in self.mixers:
            self.at_in.append(n)
            rows.append(m.rows)
            n += m.rows.shape[0]
            if n % 16:  # (every mixer's columns start at whole vectors)
                rows.append(m.rows.new_zeros(16 - n % 16, m.rows.shape[1]))
                n = pad_to(n, 16)
        n = 0
        for m in self.mixers:
            self.at_out.append(n)
            outs.append(m.w_out)
            n += m.width
        if mlp is not None:
            self.at_out.append(n)
            outs.append(torch.cat([mlp.w_out, mlp.w_out.new_zeros(mlp.w_out.shape[0], mlp.fp - mlp.w_out.shape[1])], 1))
            n += mlp.fp
        self.cols = n
        self.proj, self.o = PackedLinear(torch.cat(rows), dtype, device), PackedLinear(torch.cat(outs, 1), dtype, device)
        self.bias = self.mixers[0].out_bias
        for m in self.mixers + ([mlp] if mlp else []):
            m.rows = m.w_out = None  # (packed here)

    def tensors(self):
        own = [t for m in self.mixers if hasattr(m, "tensors") for t in m.tensors()]
        return [self.proj.w, self.o.w] + own + (self.mlp.tensors() if self.mlp else [])

    def __call__(self, h, meta: StepMeta, caches, room: AttentionRoom, side: Optional[SideStreams] = None):
        """`side`: streams 1 .. for the mixers behind the first, 0 for the feed-forward."""
        out = torch.empty(h.shape[0], self.o.K, dtype=self.dtype, device=self.device)
        if self.cols < self.o.K:
            out[:, self.cols:].zero_()

        def mix():
            x = self.proj(h)
            each = [lambda m=m, a=a, b=b, c=c: m(x[:, a:], out[:, b:b + m.width], meta, c, room)
                    for m, a, b, c in zip(self.mixers, self.at_in, self.at_out, caches)]
            run(*each, at=1)

        def feed():
            self.mlp.activate(h, out[:, self.at_out[-1]:self.at_out[-1] + self.mlp.fp])
        run = side.run if side is not None else lambda *fs, at=0: [f() for f in fs]
        run(mix, *([feed] if self.mlp is not None else []))
        return self.o(out), 1, None, self.bias


def _pack_gate_up(gate, up, fp: int, dk: int, dtype, device):
    g = torch.zeros(2, 1, fp, dk, dtype=dtype, device=device)
    f, d = gate.shape
    g[0, 0, :f, :d], g[1, 0, :f, :d] = gate.to(device), up.to(device)
    return ops.pack_groups(ops.interleave_gate_up(g[0], g[1]), dtype)


class GatedMLP:
    """down(act(gate h) * up h): the gate and up rows interleaved in one grouped projection of one group."""

    # 16-row tiles (each streams the weights) up to this many rows, by weights that passes find in the caches again
    ROWS_16, ROWS_16_LARGE, LARGE = 80, 40, 1 << 26

    def __init__(self, spec: DenseSpec, t: Dict[str, torch.Tensor], width: int, dtype, device, alone: bool = True):
        self.spec, self.dtype, self.device = spec, dtype, device
        self.dk, self.fp = pad_to(width, 64), pad_to(spec.ff, 64)
        self.w_out = t["down"]
        self.down = PackedLinear(self.w_out, dtype, device) if alone else None  # (else a MixerBlock's)
        self.w13 = _pack_gate_up(t["gate"], t["up"], self.fp, self.dk, dtype, device)
        self._tiles: Dict[int, tuple] = {}

    def tensors(self):
        return [self.w13] + ([self.down.w] if self.down else [])

    def activate(self, h, act):
        T = h.shape[0]
        if T not in self._tiles:  # (before graph capture: the capture's warm-up runs come first)
            few = self.ROWS_16 if self.w13.numel() <= self.LARGE else self.ROWS_16_LARGE
            tm = expert_tile_rows(T, self.dtype, self.dk, few, few)
            tiles = torch.tensor([[0, i, min(tm, T - i), 0] for i in range(0, T, tm)], dtype=torch.int32)
            self._tiles[T] = (tiles.to(self.device), torch.tensor([len(tiles)], dtype=torch.int32, device=self.device),
                              torch.arange(T, dtype=torch.int32, device=self.device), tm)
        tiles, n, order, tm = self._tiles[T]
        ops.expert_gemm(h, self.w13, act, tiles, n, order, T, x_div=0, out_order=False, tm=tm, glu=self.spec.act)

    def __call__(self, h, meta: StepMeta):
        act = torch.empty(h.shape[0], self.fp, dtype=self.dtype, device=self.device)
        self.activate(h, act)
        return self.down(act), 1, None, None


class PolyMLP:
    """down(polynomial norm(up h))."""

    def __init__(self, spec: PolySpec, t: Dict[str, torch.Tensor], eps: float, dtype, device):
        self.spec, self.eps = spec, eps
        self.up, self.down = PackedLinear(t["up"], dtype, device), PackedLinear(t["down"], dtype, device)
        self.act = t["act"].float().to(device).contiguous()

    def tensors(self):
        return [self.up.w, self.down.w]

    def __call__(self, h, meta: StepMeta):
        z = self.up(h)[:, :self.down.K]
        return self.down(ops.poly_norm(z, self.spec.ff, self.act, self.eps)), 1, None, None


class ScoredExperts:
    """Experts chosen by the scores of a router, and a shared expert whose pieces are further experts that
    every token uses; one partial output per (token, expert) with its weight."""

    ROWS_64, ROWS_256 = 32, 96  # average rows per expert above which they go in tiles of 64 / 256

    def __init__(self, spec: ScoredExpertsSpec, t: Dict[str, torch.Tensor], width: int, dtype, device):
        s = self.spec = spec
        self.dtype, self.device = dtype, device
        f, dk, dn = s.ff, pad_to(width, 64), pad_to(width, 128)
        # (the 256-row tiles take whole 128 columns: of a gated pair those are 64 outputs)
        self.fp, self.dk, self.dn = pad_to(f, 64 if s.act or f <= 64 else 128), dk, dn
        w13, w2 = [], []

        def add(gate, up, down):
            if gate is not None:
                w13.append(_pack_gate_up(gate, up, self.fp, dk, dtype, device))
            else:
                w = torch.zeros(1, self.fp, dk, dtype=dtype, device=device)
                w[0, :up.shape[0], :width] = up.to(device)
                w13.append(ops.pack_groups(w, dtype))
            w = torch.zeros(1, dn, self.fp, dtype=dtype, device=device)
            w[0, :width, :down.shape[1]] = down.to(device)
            w2.append(ops.pack_groups(w, dtype))
        for e in range(s.experts):
            add(t.get(f"e{e}.gate"), t[f"e{e}.up"], t[f"e{e}.down"])
        for i in range(s.always):
            a, b = i * f, min((i + 1) * f, s.shared_ff)
            add(t["shared.gate"][a:b] if s.act else None, t["shared.up"][a:b], t["shared.down"][:, a:b])
        self.w13, self.w2 = torch.cat(w13), torch.cat(w2)
        r = torch.zeros(1, pad_to(s.experts, 16), dk, dtype=dtype, device=device)
        r[0, :s.experts, :width] = t["router"].to(device)
        self.router = ops.pack_groups(r, dtype)
        self.correction = t["correction"].float().to(device).contiguous() if s.correction else None

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
                        s.groups, s.keep, s.always, tm, softmax=s.softmax, correction=self.correction, share=s.share, scale=s.scale)
        act = torch.empty(rows, self.fp, dtype=self.dtype, device=dev)
        ops.expert_gemm(h, self.w13, act, tiles, n_tiles, order, rows, x_div=K, out_order=False, tm=tm, glu=s.act,
                        relu2=s.act is None, row_w=weights if s.weigh_input else None)
        y = torch.empty(rows, self.dn, dtype=self.dtype, device=dev)
        ops.expert_gemm(act, self.w2, y, tiles, n_tiles, order, rows, x_div=0, out_order=True, tm=tm)
        return y, K, None if s.weigh_input else weights, None


class HybridModel:
    """What the engine asks of every model, for decoders of MixerBlocks: `self.layers` holds a dict per layer with
    its "mixer" block, `self.runs` the layers of a step in the order they run."""

    # the engine's decode-sized steps (EngineConfig attention settings of the Llama kernels do not apply)
    DECODE_FUSED_MAX_T = 16
    MID_MAX_T = 256
    PREFILL_MAX_T = 1 << 30
    ATT_DECODE_WAVES = 4
    PF_MIDRANGE = frozenset()
    decode_packed = True
    KERNELS = "hybrid"  # the module of its kernels (_build.py)
    ATT_HANDOFF = False  # partials are merged by a launch of their own: ordinary memory
    NAME = ""

    def __init__(self, cfg, device, dtype, tp: Optional[TPGroup], attention: Sequence[AttentionSpec], max_len: int):
        self.cfg, self.device, self.dtype = cfg, torch.device(device), dtype
        self.tp = tp or TPGroup.single()
        if self.tp.size > 1:
            raise ValueError(f"{self.NAME} models run on one GPU: tensor parallelism is not implemented for them")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"unsupported dtype {dtype}")
        if self.device.type == "cuda":  # (operations that several modules hold come from the one that is loaded)
            ops.require_family(self.KERNELS)
        self.v_local, self.vocab_offset = cfg.vocab_size, 0
        self.attention = list(attention)
        self._group = min(max([m.group for m in self.attention], default=1), 16)
        self._kv_heads = min([m.kv_heads * m.maps for m in self.attention], default=1)
        self.dec_tokens, self.tile_tokens = 16 // self._group, 128 // self._group  # tokens of an attention work item
        self._max_slots = 0
        self._max_len, self._angles = int(max_len), {}
        self.layers: List[dict] = []
        self.embed = self.head = None

    def angles(self, m: AttentionSpec):
        if m.rot_dims == 0:
            return None
        if m.rotation not in self._angles:
            self._angles[m.rotation] = m.angles(self._max_len).to(self.device)
        return self._angles[m.rotation]

    def f32(self, t: torch.Tensor) -> torch.Tensor:
        return t.float().to(self.device).contiguous()

    def weights(self, path: Optional[str], draw, seed: int):
        """get(name, shape): the folder's tensors, or draw(name behind the layer, an empty tensor, a generator)."""
        if path:
            return checkpoint_reader(path)
        g = torch.Generator(device=self.device).manual_seed(seed)
        return lambda name, shape: draw(name.split(".", 1)[-1], torch.empty(shape, dtype=torch.bfloat16, device=self.device), g)

    def finish(self) -> None:
        if self.device.type == "cuda" and self.dtype == torch.bfloat16:  # before any graph capture
            ops.decode_workspace(self.device)
            ops.prefill_workspace(self.device)

    def weight_bytes(self) -> int:
        ts = [self.embed, self.head.w]
        for L in self.layers:
            ts += L["mixer"].tensors() + (L["mlp"].tensors() if L["mlp"] else [])
        return sum(t.numel() * t.element_size() for t in ts)

    def _kinds(self) -> List[List[tuple]]:
        return [[m.cache_kind() for m in self.layers[i]["mixer"].mixers] for i in self.runs]

    def cache_bytes_per_block(self, block_size: int) -> int:
        return HybridCache.bytes_per_block(self._kinds(), self.embed.element_size(), block_size)

    def state_bytes_per_slot(self) -> int:
        return HybridCache.bytes_per_slot(self._kinds(), self.embed.element_size())

    def make_cache(self, num_blocks: int, block_size: int, slots: int = 0) -> HybridCache:
        return HybridCache(self._kinds(), num_blocks, slots, self.device, self.dtype, block_size)

    def attention_items(self) -> dict:
        keys = [m.max_keys for m in self.attention]
        pools = [m.pool for m in self.attention if m.pool]
        out = {"gqa_group": self._group, "kv_heads": self._kv_heads, "att_qcols": 128, "att_narrow_qcols": 128,
               "prefill_split_keys": 0, "decode_part_target": 256, "att_min_part": 256,
               "att_tile_target": max(16, 256 // self._kv_heads), "att_max_keys": max(keys) if keys and all(keys) else 0,
               "att_pool": min(pools, default=0)}
        if self.state_bytes_per_slot():  # a page's worth of state is not kept, so a prefix cannot be taken from the cache
            out.update(scan_chunk=ops.SCAN_CHUNK, scan_min=ops.SCAN_MIN, prefix_caching=False)
        return out

    def attention_workspace(self, max_items: int) -> tuple:
        """(partial outputs, partial (max, sum) pairs) in floats, and tickets per sequence (none)."""
        self._max_slots = max_items
        o = ml = 1
        for m in self.attention:
            n = max_items * m.kv_heads * m.maps * ((self.dec_tokens * m.group + 15) // 16) * 16
            o, ml = max(o, n * m.out_width), max(ml, n * 2)
        return o, ml, 1

    def room(self, part_o, part_ml) -> AttentionRoom:
        return AttentionRoom(part_o, part_ml, self.dec_tokens, self.tile_tokens, self._max_slots)

    def health_words(self) -> list:
        return []

    def into_pool(self, hn: torch.Tensor, embed: tuple) -> None:
        """Embedding requests: their rows of the last norm's output join the pool (see LlamaModel.forward)."""
        pool_rows, pool = embed
        pool[-1].zero_()  # the row of tokens that no embedding request owns
        pool.index_add_(0, pool_rows[:hn.shape[0]].long(), hn[:, :self.cfg.hidden_size].float())
