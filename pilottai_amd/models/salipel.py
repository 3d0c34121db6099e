"""Salipel: a decoder of parallel blocks, whose mixer and feed-forward read one norm of the residual, with mixers of
three types in any order.

    x = E[token];   per layer  h = norm(x),  x <- x + m (mixer(h) + ff(h));   logits = W norm(x)

  parallel     windowed attention whose values are the projected keys, beside a matrix memory (mLSTM); their weighted
               sum. Normed and rotated queries and keys, kept first tokens, an output gate.
  attention    attention within chunks of positions, without rotation: a bias by distance, normed values, a learned
               sink per head
  attention_2  differential attention: two maps per head over the same values; normed and rotated queries and keys,
               capped scores, an output gate

Feed-forwards: gated (tanh gelu), experts (square of relu) chosen by softmax scores with a correction, or none.
norm(u) = u / rms(u) w. The residual, norms, rotations, scores, softmax, router, gates and state of the recurrence
are fp32; activations and matrix products are the model's dtype (bf16, or fp32 throughout).

One step of T tokens (decode rows and prompt portions alike), sublayers in models/hybrid.py:

  once      hyper_norm          x = E[id], norm -> h (one stream)
  mixer     linear              every mixer's projections of h in one matrix
            paged_kv            head norms, rotation, paged keys and values
            window_attention    with its gate; or both maps, then head_difference with the gate
            matrix_memory       decode rows in one launch; longer portions in chunks; gated_norm
  dense     expert_gemm         gate and up of one group, gated, beside the mixer's output
  experts   score_route, expert_gemm x 2
  output    linear              the mixers' output matrices and the dense second one as one product
  between   hyper_norm          m times the output and the weighted experts into x, next norm -> h
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional, Tuple, Union

import torch

from pilottai_amd import ops
from pilottai_amd.models.cache import HybridCache, StepMeta
from pilottai_amd.models.common import PackedLinear
from pilottai_amd.models.hybrid import (GELU_TANH, AttentionSpec, DenseSpec, GatedMLP, HybridModel, MatrixMemory, MatrixMemorySpec,
                                        MixerBlock, PagedAttention, ScoredExperts, ScoredExpertsSpec, SideStreams)
from pilottai_amd.ops.latent import pad_to
from pilottai_amd.parallel.comm import TPGroup


@dataclass(frozen=True)
class ParallelSpec:
    """A windowed attention and a matrix memory side by side."""
    left: AttentionSpec
    right: MatrixMemorySpec
    left_scale: float
    right_scale: float

    def shapes(self, d: int) -> Dict[str, tuple]:
        return {f"{side}.{k}": s for side, m in (("left", self.left), ("right", self.right)) for k, s in m.shapes(d).items()}


@dataclass(frozen=True)
class SalipelLayer:
    mixer: Union[AttentionSpec, ParallelSpec]
    mlp: Union[DenseSpec, ScoredExpertsSpec, None]


def _sizes(m: dict) -> dict:
    return dict(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), scale=float(m["scale"]))


def _rotation(rot: dict) -> dict:
    sc = rot.get("scaling")
    return dict(rot_base=float(rot["base"]), rot_dims=int(rot["dims"]),
                slow_waves=tuple(float(sc[k]) for k in ("factor", "low", "high", "original")) if sc else None)


def _window(m: dict) -> AttentionSpec:
    mask = m.get("mask") or {}
    return AttentionSpec(**_sizes(m), **_rotation(m["rot"]), window=int(mask.get("size") or 0),
                         keep=int(mask.get("keep_first") or 0) if mask.get("size") else 0, qk_norm=True, keys_as_values=True,
                         gate=True)


def _parallel(m: dict) -> ParallelSpec:
    r = m["right"]
    return ParallelSpec(_window(m["left"]), MatrixMemorySpec(int(r["heads"]), int(r["dim"]), int(r["vdim"]), float(r["gate_cap"])),
                        float(m["left_scale"]), float(m["right_scale"]))


def distance_slopes(heads: int) -> Tuple[float, ...]:
    return tuple(2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads))


def _chunked(m: dict) -> AttentionSpec:
    return AttentionSpec(**_sizes(m), chunk=int((m.get("mask") or {}).get("size") or 0), slopes=distance_slopes(int(m["heads"])),
                         learned_sink=True, v_norm=True)


def _differential(m: dict) -> AttentionSpec:
    return AttentionSpec(**_sizes(m), **_rotation(m["rot"]), cap=float(m.get("softcap") or 0.0), diff=float(m["diff"]), qk_norm=True,
                         gate=True)


def _feed_forward(p: Optional[dict]):
    if p is None:
        return None
    if p.get("kind") == "dense":
        return DenseSpec(int(p["ff"]), GELU_TANH)
    if p.get("kind") != "moe":
        raise ValueError(f"unknown feed-forward {p.get('kind')!r}")
    r = p["router"]
    return ScoredExpertsSpec(experts=int(r["experts"]), top=int(r["top"]), ff=int(p["expert"]["ff"]), act=None, softmax=True,
                             correction=True, share=True, scale=float(r.get("scale", 1.0)))


MIXERS = {"parallel": _parallel, "attention": _chunked, "attention_2": _differential}


@dataclass
class SalipelConfig:
    name: str
    vocab_size: int
    hidden_size: int
    layers: List[SalipelLayer]
    eps: float = 1e-5
    residual_mult: float = 1.0
    max_position: int = 1 << 20
    init_std: float = 0.02

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def runs(self) -> List[int]:
        """The layers of a step in the order they run."""
        return list(range(self.num_layers))

    @classmethod
    def from_dict(cls, d: dict, name: str = "salipel") -> "SalipelConfig":
        layers = []
        for i, L in enumerate(d["layers"]):
            if L.get("type") not in MIXERS:
                raise ValueError(f"layer {i}: unknown mixer {L.get('type')!r}")
            try:
                layers.append(SalipelLayer(MIXERS[L["type"]](L["mixer"]), _feed_forward(L.get("mlp"))))
            except ValueError as e:
                raise ValueError(f"layer {i}: {e}") from None
        return cls(name=name, vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), layers=layers,
                   eps=float(d["norm"]["eps"]), residual_mult=float(d.get("residual_mult", 1.0)))

    def layer_shapes(self, i: int) -> Dict[str, tuple]:
        """Every tensor of layer i by its name behind "l<i>."."""
        L, d = self.layers[i], self.hidden_size
        out: Dict[str, tuple] = {"norm1": (d,)}
        for pre, spec in (("mix.", L.mixer), ("mlp.", L.mlp)):
            if spec is not None:
                out.update({pre + k: s for k, s in spec.shapes(d).items()})
        return out

    def num_params(self) -> int:
        size = lambda s: torch.Size(s).numel()  # noqa: E731
        return (2 * self.vocab_size + 1) * self.hidden_size + sum(size(s) for i in range(self.num_layers)
                                                                  for s in self.layer_shapes(i).values())


def _preset(name: str, width: int, heads: int, memory: MatrixMemorySpec, ff: int, experts: ScoredExpertsSpec, repeat: int,
            vocab: int = 128256) -> SalipelConfig:
    """Layers of a real model's size: heads of 128, a quarter of them as KV heads."""
    size = dict(heads=heads, kv_heads=heads // 4, vdim=128)
    left = AttentionSpec(**size, dim=128, scale=128 ** -0.5, rot_base=500000.0, rot_dims=128, slow_waves=(8.0, 1.0, 4.0, 8192.0),
                         window=1024, keep=16, qk_norm=True, keys_as_values=True, gate=True)
    chunked = AttentionSpec(**size, dim=128, scale=128 ** -0.5, chunk=2048, slopes=distance_slopes(heads), learned_sink=True,
                            v_norm=True)
    twice = AttentionSpec(**size, dim=64, scale=64 ** -0.5, rot_base=500000.0, rot_dims=64, cap=50.0, diff=0.4, qk_norm=True, gate=True)
    both = ParallelSpec(left, memory, 1.0, 1.0)
    layers = [SalipelLayer(chunked, DenseSpec(ff)), SalipelLayer(both, experts), SalipelLayer(twice, DenseSpec(ff)),
              SalipelLayer(both, experts)]
    return SalipelConfig(name=name, vocab_size=vocab, hidden_size=width, layers=layers * repeat, residual_mult=0.5)


def _experts(n: int, top: int, ff: int) -> ScoredExpertsSpec:
    return ScoredExpertsSpec(experts=n, top=top, ff=ff, act=None, softmax=True, correction=True, share=True, scale=2.0)


PRESETS: Dict[str, SalipelConfig] = {
    # a small shape for tests of the engine around the model (the tokenizer's vocabulary)
    "salipel-tiny": SalipelConfig("salipel-tiny", 128256, 160, [
        SalipelLayer(AttentionSpec(6, 2, 40, 24, 0.2, chunk=50, slopes=distance_slopes(6), learned_sink=True, v_norm=True),
                     _experts(6, 2, 72)),
        SalipelLayer(ParallelSpec(AttentionSpec(3, 1, 48, 48, 0.2, 10000.0, 32, window=70, keep=5, qk_norm=True,
                                                keys_as_values=True, gate=True), MatrixMemorySpec(4, 24, 40, 15.0), 0.9, 1.2),
                     DenseSpec(200)),
        SalipelLayer(AttentionSpec(4, 2, 24, 40, 0.3, 10000.0, 24, cap=30.0, diff=0.4, qk_norm=True, gate=True), None)]),
    # layers of a real model's size (bench.py --design salipel), at two widths
    "salipel-base": _preset("salipel-base", 2048, 16, MatrixMemorySpec(8, 128, 256, 15.0), 8192, _experts(64, 6, 1408), 2),
    "salipel-wide": _preset("salipel-wide", 4096, 32, MatrixMemorySpec(16, 128, 256, 15.0), 14336, _experts(64, 6, 2048), 1),
}


class SalipelModel(HybridModel):
    NAME = "Salipel"
    SIDE_MAX_T = 2048  # largest captured step whose feed-forward and second mixer run beside the first mixer

    def __init__(self, cfg: SalipelConfig, device, dtype=torch.bfloat16, tp: Optional[TPGroup] = None, seed: int = 0,
                 weights_path: Optional[str] = None, max_len: int = 8192, **_):
        attention = [m.left if isinstance(m, ParallelSpec) else m for m in (L.mixer for L in cfg.layers)]
        super().__init__(cfg, device, dtype, tp, attention, max_len)
        self.runs = cfg.runs()
        get = self.weights(weights_path, self._draw, seed)
        d, V, dev = cfg.hidden_size, cfg.vocab_size, self.device
        self.embed = get("embed", (V, d)).to(dev, dtype).contiguous()
        self.head = PackedLinear(get("head", (V, d)), dtype, dev)
        self.norm = self.f32(get("final.norm", (d,)))
        self.one = torch.ones(1, dtype=torch.float32, device=dev)
        self.keep, self.mult = torch.ones(1, 1, dtype=torch.float32, device=dev), self.one * cfg.residual_mult
        for i, L in enumerate(cfg.layers):
            t = {k: get(f"l{i}.{k}", s) for k, s in cfg.layer_shapes(i).items()}
            sub = lambda pre: {k[len(pre):]: v for k, v in t.items() if k.startswith(pre)}  # noqa: E731, B023
            m = L.mixer
            if isinstance(m, ParallelSpec):
                mixers = [PagedAttention(m.left, sub("mix.left."), dtype, dev, self.angles(m.left), cfg.eps, m.left_scale),
                          MatrixMemory(m.right, sub("mix.right."), cfg.eps, dtype, dev, m.right_scale)]
            else:
                mixers = [PagedAttention(m, sub("mix."), dtype, dev, self.angles(m), cfg.eps)]
            dense = GatedMLP(L.mlp, sub("mlp."), d, dtype, dev, alone=False) if isinstance(L.mlp, DenseSpec) else None
            experts = ScoredExperts(L.mlp, sub("mlp."), d, dtype, dev) if isinstance(L.mlp, ScoredExpertsSpec) else None
            self.layers.append({"norm": self.f32(t["norm1"]), "mixer": MixerBlock(mixers, dtype, dev, dense), "mlp": experts})
        self.side = SideStreams(dev, 2)
        self.finish()

    def _draw(self, part: str, rand: torch.Tensor, g: torch.Generator):
        if part == "norm" or part.endswith((".norm", "norm1")):
            return rand.fill_(1.0)
        if part.endswith((".sink", ".correction", ".i.b")):
            return rand.zero_()
        if part.endswith(".f.b"):  # forget gates near 1, as the memories start
            return rand.copy_(torch.linspace(3.0, 6.0, rand.shape[0], device=rand.device))
        return rand.normal_(0.0, self.cfg.init_std, generator=g)

    # -- forward -----------------------------------------------------------------
    def forward(self, meta: StepMeta, kv: HybridCache, num_tokens: int, num_logit_rows: int, part_o: torch.Tensor,
                part_ml: torch.Tensor, embed=None, residuals: Optional[list] = None) -> torch.Tensor:
        """Logits [num_logit_rows, vocab] of rows meta.logit_rows. embed = (rows, pool): see
        LlamaModel.forward. `residuals` (a list) collects the residual after every layer."""
        cfg, T, dev = self.cfg, num_tokens, self.device
        eps, d = cfg.eps, cfg.hidden_size
        new_h = lambda n=T: torch.empty(n, pad_to(d, 64), dtype=self.dtype, device=dev)  # noqa: E731
        x = torch.empty(T, 1, d, dtype=torch.float32, device=dev)  # one stream
        room = self.room(part_o, part_ml)
        step = dict(emb=self.embed, ids=meta.input_ids[:T])
        for i, L in enumerate(self.layers):
            h = ops.hyper_norm(x, eps, pre=self.one, w_next=L["norm"], out=new_h(), **step)
            side = self.side if T <= self.SIDE_MAX_T else None
            mixer, mlp = lambda: L["mixer"](h, meta, kv.layers[i], room, side), lambda: L["mlp"](h, meta)  # noqa: E731, B023
            both = [mixer] + ([mlp] if L["mlp"] is not None else [])
            (y, *_), *more = side.run(*both) if side else [f() for f in both]
            step = dict(y=y, mix=self.keep, post=self.mult)
            if more:
                part, k, w, _ = more[0]
                step.update(y=part, partials=k, y_weights=w, y2=y)
            if residuals is not None:
                after = x.clone()
                ops.hyper_norm(after, eps, **step)
                residuals.append(after[:, 0])
        final = dict(pre=self.one, w_next=self.norm)
        if embed is not None:
            self.into_pool(ops.hyper_norm(x, eps, out=new_h(), **final, **step), embed)
            step = {}
        hs = ops.hyper_norm(x, eps, out=new_h(num_logit_rows), rows=meta.logit_rows[:num_logit_rows], **final, **step)
        return self.head(hs)[:, :cfg.vocab_size]
