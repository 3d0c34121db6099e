"""Mudepel: a decoder whose residual has several streams (hyper-connections) and whose layers mix windowed
attention over tokens and pooled blocks with Mamba-2, and dense with score-routed feed-forwards, in a
looped stack.

    x_1 .. x_S = E[token]
    per sublayer:   u = sum_s in[s] x_s,  y = sublayer(norm(u)),  x_t <- sum_s mix[s, t] x_s + out[t] y
    logits = cap tanh(E . norm(sum_s x_s) / cap)

norm(u) = u / rms(u) (1 + w). A loop runs layers start .. stop-1 `times` times with the same weights;
every pass has its own cache pools and state slots (models/cache.py HybridCache).

The streams, norms, rotations, scores, softmax, router sums and the recurrence are fp32; activations and
matrix products are the model's dtype (bf16, or fp32 throughout).

One step of T tokens (decode rows and prompt portions alike), sublayers in models/hybrid.py:

  once        hyper_norm        x = E[id], norm -> h
  attention   linear            q | k | v, one projection
              paged_kv          biases, rotation, paged keys and values, pooled blocks that end here
              window_attention  tokens and blocks in one softmax; merge of partitions
              linear
  mamba2      linear            z | x | B | C | dt, one projection
              state_scan        decode rows with their convolution in one launch; longer portions in chunks
              gated_norm, linear
  dense       expert_gemm       gate and up of one group, gated; linear
  experts     score_route       choices, weights, rows sorted by expert, the shared expert among them
              expert_gemm x 2   one partial output per (token, expert)
  between     hyper_norm        weighted partials + bias into the streams, next norm -> h
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional, Tuple, Union

import torch

from pilottai_amd import ops
from pilottai_amd.models.cache import HybridCache, StepMeta
from pilottai_amd.models.common import PackedLinear, layer_runs, parse_loop
from pilottai_amd.models.hybrid import (AttentionSpec, DenseSpec, GatedMLP, HybridModel, MixerBlock, PagedAttention, ScoredExperts,
                                        ScoredExpertsSpec, StateSpace, StateSpaceSpec)
from pilottai_amd.ops.latent import pad_to
from pilottai_amd.parallel.comm import TPGroup


@dataclass(frozen=True)
class MudepelLayer:
    mixer: Union[AttentionSpec, StateSpaceSpec]
    mlp: Union[DenseSpec, ScoredExpertsSpec, None]


def _attention(m: dict) -> AttentionSpec:
    rot, mask = m["rot"], m.get("mask") or {}
    sc = rot.get("scaling")
    return AttentionSpec(
        heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), scale=float(m["scale"]),
        rot_base=float(rot["base"]), rot_dims=int(rot["dims"]),
        yarn=tuple(float(sc[k]) for k in ("factor", "original", "fast", "slow")) if sc else None,
        window=int(mask.get("size") or 0), pool=int(mask.get("pool") or 0), sink=1.0, bias=True)


def _mamba2(m: dict) -> StateSpaceSpec:
    spec = StateSpaceSpec(**{k: int(m[k]) for k in ("heads", "vdim", "state", "groups", "conv", "norm_groups")})
    if spec.heads % spec.groups or spec.heads * spec.vdim % spec.norm_groups:
        raise ValueError(f"{spec.heads} heads of {spec.vdim} do not divide into {spec.groups} groups, "
                         f"{spec.norm_groups} normed parts")
    return spec


def _feed_forward(p: Optional[dict]):
    if p is None:
        return None
    if p.get("kind") == "dense":
        return DenseSpec(int(p["ff"]))
    if p.get("kind") != "moe":
        raise ValueError(f"unknown feed-forward {p.get('kind')!r}")
    r = p["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    return ScoredExpertsSpec(experts=int(r["experts"]), top=int(r["top"]), ff=int(p["expert"]["ff"]), groups=int(g["count"]),
                             keep=int(g["keep"]), shared_ff=int(p["shared"]["ff"]) if p.get("shared") else 0)


@dataclass
class MudepelConfig:
    name: str
    vocab_size: int
    hidden_size: int
    layers: List[MudepelLayer]
    streams: int = 1
    eps: float = 1e-5
    softcap: float = 0.0  # of the logits; 0: none
    loop: Optional[Tuple[int, int, int]] = None  # (start, stop, times)
    max_position: int = 1 << 20
    init_std: float = 0.02

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def runs(self) -> List[int]:
        """The layers of a step in the order they run."""
        return [i for i, _ in layer_runs(self.num_layers, self.loop)]

    @classmethod
    def from_dict(cls, d: dict, name: str = "mudepel") -> "MudepelConfig":
        mixers = {"attention": _attention, "mamba2": _mamba2}
        layers = []
        for i, L in enumerate(d["layers"]):
            if L.get("type") not in mixers:
                raise ValueError(f"layer {i}: unknown mixer {L.get('type')!r}")
            try:
                layers.append(MudepelLayer(mixers[L["type"]](L["mixer"]), _feed_forward(L.get("mlp"))))
            except ValueError as e:
                raise ValueError(f"layer {i}: {e}") from None
        return cls(name=name, vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), layers=layers,
                   streams=int(d.get("streams") or 1), eps=float(d["norm"]["eps"]),
                   softcap=float(d.get("logit_softcap") or 0.0), loop=parse_loop(d.get("loop"), len(layers)))

    def layer_shapes(self, i: int) -> Dict[str, tuple]:
        """Every tensor of layer i by its name behind "l<i>."."""
        L, d, S = self.layers[i], self.hidden_size, self.streams
        subs = [("norm1", "hc1.", "mix.", L.mixer)] + ([("norm2", "hc2.", "mlp.", L.mlp)] if L.mlp else [])
        out: Dict[str, tuple] = {}
        for norm, hc, pre, spec in subs:
            out[norm] = (d,)
            out.update({hc + "in": (S,), hc + "out": (S,), hc + "mix": (S, S)})
            out.update({pre + k: s for k, s in spec.shapes(d).items()})
        return out

    def num_params(self) -> int:
        size = lambda s: torch.Size(s).numel()  # noqa: E731
        return (self.vocab_size + 1) * self.hidden_size + sum(size(s) for i in range(self.num_layers)
                                                              for s in self.layer_shapes(i).values())


def _alternating(name: str, width: int, pairs: int, att: AttentionSpec, ssm: StateSpaceSpec, dense: DenseSpec,
                 moe: ScoredExpertsSpec, streams: int, vocab: int = 128256, loop=None) -> MudepelConfig:
    return MudepelConfig(name=name, vocab_size=vocab, hidden_size=width, streams=streams, softcap=30.0, loop=loop,
                         layers=[MudepelLayer(att, dense), MudepelLayer(ssm, moe)] * pairs)


PRESETS: Dict[str, MudepelConfig] = {
    # a small shape for tests of the engine around the model (the tokenizer's vocabulary)
    "mudepel-tiny": _alternating("mudepel-tiny", 160, 1,
                                 AttentionSpec(heads=6, kv_heads=2, dim=40, vdim=24, scale=0.2, rot_base=10000.0,
                                               rot_dims=32, window=150, pool=10, sink=1.0, bias=True),
                                 StateSpaceSpec(heads=4, vdim=40, state=24, groups=2, conv=4, norm_groups=2), DenseSpec(200),
                                 ScoredExpertsSpec(experts=6, top=2, ff=72, groups=3, keep=2, shared_ff=80), 2,
                                 loop=(0, 1, 2)),
    # layers of a real model's size (bench.py --design mudepel), at two widths
    "mudepel-base": _alternating("mudepel-base", 2048, 4,
                                 AttentionSpec(heads=16, kv_heads=4, dim=128, vdim=128, scale=128 ** -0.5,
                                               rot_base=500000.0, rot_dims=128, yarn=(4.0, 8192.0, 32.0, 1.0),
                                               window=2048, pool=16, sink=1.0, bias=True),
                                 StateSpaceSpec(heads=64, vdim=64, state=128, groups=8, conv=4, norm_groups=8),
                                 DenseSpec(8192), ScoredExpertsSpec(experts=64, top=6, ff=1408, groups=8, keep=4,
                                                                    shared_ff=1408), 4),
    "mudepel-wide": _alternating("mudepel-wide", 4096, 2,
                                 AttentionSpec(heads=32, kv_heads=8, dim=128, vdim=128, scale=128 ** -0.5,
                                               rot_base=500000.0, rot_dims=128, yarn=(4.0, 8192.0, 32.0, 1.0),
                                               window=2048, pool=16, sink=1.0, bias=True),
                                 StateSpaceSpec(heads=128, vdim=64, state=128, groups=8, conv=4, norm_groups=8),
                                 DenseSpec(14336), ScoredExpertsSpec(experts=64, top=6, ff=2048, groups=8, keep=4,
                                                                     shared_ff=2048), 4),
}


class MudepelModel(HybridModel):
    NAME = "Mudepel"

    def __init__(self, cfg: MudepelConfig, device, dtype=torch.bfloat16, tp: Optional[TPGroup] = None, seed: int = 0,
                 weights_path: Optional[str] = None, max_len: int = 8192, **_):
        super().__init__(cfg, device, dtype, tp, [L.mixer for L in cfg.layers if isinstance(L.mixer, AttentionSpec)], max_len)
        self.runs = cfg.runs()
        get = self.weights(weights_path, self._draw, seed)
        d, dev, f32 = cfg.hidden_size, self.device, self.f32
        embed = get("embed", (cfg.vocab_size, d))
        self.embed = embed.to(dev, dtype).contiguous()
        self.head = PackedLinear(embed, dtype, dev)
        self.norm = f32(1 + get("final.norm", (d,)).float())
        self.ones = torch.ones(cfg.streams, dtype=torch.float32, device=dev)
        for i, L in enumerate(cfg.layers):
            t = {k: get(f"l{i}.{k}", s) for k, s in cfg.layer_shapes(i).items()}
            sub = lambda pre: {k[len(pre):]: v for k, v in t.items() if k.startswith(pre)}  # noqa: E731, B023
            if isinstance(L.mixer, AttentionSpec):
                mixer = PagedAttention(L.mixer, sub("mix."), dtype, dev, self.angles(L.mixer))
            else:
                mixer = StateSpace(L.mixer, sub("mix."), cfg.eps, dtype, dev)
            mlp = None
            if L.mlp is not None:
                mlp = (GatedMLP if isinstance(L.mlp, DenseSpec) else ScoredExperts)(L.mlp, sub("mlp."), d, dtype, dev)
            layer = {"mixer": MixerBlock([mixer], dtype, dev), "mlp": mlp}
            for q in (1, 2) if mlp else (1,):
                layer[f"norm{q}"] = f32(1 + t[f"norm{q}"].float())
                layer[f"hc{q}"] = {k: f32(v) for k, v in sub(f"hc{q}.").items()}
            self.layers.append(layer)
        self.finish()

    def _draw(self, part: str, rand: torch.Tensor, g: torch.Generator):
        cfg, dev = self.cfg, self.device
        if part in ("hc1.in", "hc2.in"):
            return rand.fill_(1.0 / cfg.streams)
        if part in ("hc1.mix", "hc2.mix"):
            return torch.eye(cfg.streams, dtype=torch.bfloat16, device=dev)
        if part in ("hc1.out", "hc2.out", "mix.D", "mix.norm"):
            return rand.fill_(1.0)
        if part in ("norm1", "norm2", "norm", "mix.conv.b", "mix.q.b", "mix.k.b", "mix.v.b", "mix.o.b"):
            return rand.zero_()
        if part == "mix.A_log":  # decays of exp(-dt) .. exp(-16 dt)
            return torch.log(torch.linspace(1, 16, rand.shape[0], device=dev)).to(torch.bfloat16)
        if part == "mix.dt_bias":  # step sizes about 0.01
            return rand.fill_(-4.6)
        if part == "mix.conv":
            return rand.normal_(0.0, rand.shape[1] ** -0.5, generator=g)
        return rand.normal_(0.0, cfg.init_std, generator=g)

    # -- forward -----------------------------------------------------------------
    def forward(self, meta: StepMeta, kv: HybridCache, num_tokens: int, num_logit_rows: int, part_o: torch.Tensor,
                part_ml: torch.Tensor, embed=None, residuals: Optional[list] = None) -> torch.Tensor:
        """Logits [num_logit_rows, vocab] of rows meta.logit_rows. embed = (rows, pool): see
        LlamaModel.forward. `residuals` (a list) collects the sum of the streams after every layer run."""
        cfg, T, dev = self.cfg, num_tokens, self.device
        eps, d = cfg.eps, cfg.hidden_size
        ldh = pad_to(d, 64)
        new_h = lambda n=T: torch.empty(n, ldh, dtype=self.dtype, device=dev)  # noqa: E731
        x = torch.empty(T, cfg.streams, d, dtype=torch.float32, device=dev)
        step, room = dict(emb=self.embed, ids=meta.input_ids[:T]), self.room(part_o, part_ml)
        for j, i in enumerate(self.runs):
            L = self.layers[i]
            h = ops.hyper_norm(x, eps, pre=L["hc1"]["in"], w_next=L["norm1"], out=new_h(), **step)
            step = self._into_streams(L["mixer"](h, meta, kv.layers[j], room), L["hc1"])
            if L["mlp"] is not None:
                h = ops.hyper_norm(x, eps, pre=L["hc2"]["in"], w_next=L["norm2"], out=new_h(), **step)
                step = self._into_streams(L["mlp"](h, meta), L["hc2"])
            if residuals is not None:
                after = x.clone()
                ops.hyper_norm(after, eps, **step)
                residuals.append(after.sum(1))
        final = dict(pre=self.ones, w_next=self.norm)
        if embed is not None:
            self.into_pool(ops.hyper_norm(x, eps, out=new_h(), **final, **step), embed)
            step = {}
        hs = ops.hyper_norm(x, eps, out=new_h(num_logit_rows), rows=meta.logit_rows[:num_logit_rows], **final, **step)
        logits = self.head(hs)
        if cfg.softcap:
            ops.softcap(logits, cfg.vocab_size, cfg.softcap)
        return logits[:, :cfg.vocab_size]

    @staticmethod
    def _into_streams(result, hc) -> dict:
        y, partials, weights, bias = result
        return dict(y=y, partials=partials, y_weights=weights, bias=bias, mix=hc["mix"], post=hc["out"])
