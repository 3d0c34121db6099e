"""Pusunex: a decoder whose layers mix latent attention, with or without rotated positions and partly over another
layer's cache, with gated linear attention; norms in groups before and after every sublayer, a gated embedding of the token
into every layer, and averages over depth.

    x = X_0 = E[token]
    per layer i:   x += n(mixer(n(x)));  x += n(ff(n(x)));  x += rms(W_p (gelu(W_g x) * E_i[token])) w
                   X_(i+1) = x;  x = sum_j a_ij X_j
    logits = W n(x)

  latent_attention    queries straight from the input, no positions, an output gate; with `kv_from` the latents that
                      another layer has cached
  latent_attention_2  queries through a latent of their own, a rotated part (neighbouring pairs)
  gla                 gated linear attention

Feed-forwards: dense with a polynomial norm as activation, experts chosen by sigmoid scores that weigh their inputs (and a
shared expert), or none. n norms equal parts of its vector each by itself. The residual, all X_j, norms, rotations, scores,
softmax, router, decays and the recurrent state are fp32; activations and matrix products are the model's dtype (bf16, or
fp32 throughout).

One step of T tokens (decode rows and prompt portions alike), mixers in models/latent.py and hybrid.py:

  once       residual_norm       x = E[id], norm -> h
  latent     linear              [queries or query latent | kv latent | rotated key | gate], one projection
             latent_cache, head_gemm, latent_attention, head_gemm (times the gate)
  gla        linear              [q | k | v | gate | low-rank decays], one projection
             linear_attention    decode rows in one launch; longer portions in chunks; gated_norm
  output     linear
  ff         linear, poly_norm, linear; or score_route, expert_gemm x 2
  behind ff  residual_norm       x += norm(weighted partials) -> x as the next projection's input
             table_gemm          gelu(W_g x) times the token's row of E_i
             linear
             residual_norm       x += norm(y), the average over depth, the next layer's norm -> h
"""
from __future__ import annotations

from dataclasses import dataclass, replace
from typing import Dict, List, Optional, Union

import torch

from pilottai_amd import ops
from pilottai_amd.models.cache import HybridCache, StepMeta
from pilottai_amd.models.common import PackedLinear
from pilottai_amd.models.hybrid import (GELU_TANH, HybridModel, LinearAttention, LinearAttentionSpec, MixerBlock, PolyMLP, PolySpec,
                                        ScoredExperts, ScoredExpertsSpec)
from pilottai_amd.models.latent import LatentAttention, LatentAttentionSpec
from pilottai_amd.ops.latent import pad_to
from pilottai_amd.parallel.comm import TPGroup


@dataclass(frozen=True)
class PusunexLayer:
    mixer: Union[LatentAttentionSpec, LinearAttentionSpec]
    mlp: Union[PolySpec, ScoredExpertsSpec, None]


def _latent(m: dict) -> LatentAttentionSpec:
    source = m.get("kv_from")
    return LatentAttentionSpec(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), kv_rank=int(m["kv_rank"]),
                               scale=float(m["scale"]), gate=True, kv_from=None if source is None else int(source))


def _latent_rotated(m: dict) -> LatentAttentionSpec:
    rot = m["rot"]
    return LatentAttentionSpec(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), kv_rank=int(m["kv_rank"]),
                               scale=float(m["scale"]), q_rank=int(m["q_rank"]), rot_dim=int(m["rot_dim"]),
                               rot_base=float(rot["base"]), rot_dims=int(rot.get("dims", m["rot_dim"])), rot_pairs=True)


def _linear(m: dict) -> LinearAttentionSpec:
    return LinearAttentionSpec(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), tau=float(m["tau"]))


MIXERS = {"latent_attention": _latent, "latent_attention_2": _latent_rotated, "gla": _linear}


def _feed_forward(p: Optional[dict]):
    if p is None:
        return None
    if p.get("kind") == "dense":
        return PolySpec(int(p["ff"]))
    if p.get("kind") != "moe":
        raise ValueError(f"unknown feed-forward {p.get('kind')!r}")
    r = p["router"]
    return ScoredExpertsSpec(experts=int(r["experts"]), top=int(r["top"]), ff=int(p["expert"]["ff"]),
                             shared_ff=int(p["shared"]["ff"]) if p.get("shared") else 0, weigh_input=True)


@dataclass
class PusunexConfig:
    name: str
    vocab_size: int
    hidden_size: int
    layers: List[PusunexLayer]
    eps: float = 1e-5
    norm_groups: int = 1
    side_dim: int = 0  # the token's own input to a layer; 0: none
    max_position: int = 1 << 20
    init_std: float = 0.02

    def __post_init__(self):
        if self.hidden_size % self.norm_groups:
            raise ValueError(f"{self.hidden_size} dimensions do not divide into {self.norm_groups} parts")
        for i, L in enumerate(self.layers):
            j = getattr(L.mixer, "kv_from", None)
            if j is None:
                continue
            m = self.layers[j].mixer if 0 <= j < i else None
            if not isinstance(m, LatentAttentionSpec) or m.kv_from is not None or m.kv_rank != L.mixer.kv_rank:
                raise ValueError(f"layer {i}: layer {j} has no latents of size {L.mixer.kv_rank} of its own")

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def runs(self) -> List[int]:
        """The layers of a step in the order they run."""
        return list(range(self.num_layers))

    @classmethod
    def from_dict(cls, d: dict, name: str = "pusunex") -> "PusunexConfig":
        layers = []
        for i, L in enumerate(d["layers"]):
            if L.get("type") not in MIXERS:
                raise ValueError(f"layer {i}: unknown mixer {L.get('type')!r}")
            try:
                layers.append(PusunexLayer(MIXERS[L["type"]](L["mixer"]), _feed_forward(L.get("mlp"))))
            except ValueError as e:
                raise ValueError(f"layer {i}: {e}") from None
        return cls(name=name, vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), layers=layers,
                   eps=float(d["norm"]["eps"]), norm_groups=int(d["norm"].get("groups") or 1),
                   side_dim=int((d.get("token_side") or {}).get("dim") or 0))

    def layer_shapes(self, i: int) -> Dict[str, tuple]:
        """Every tensor of layer i by its name behind "l<i>."."""
        L, d, e = self.layers[i], self.hidden_size, self.side_dim
        out: Dict[str, tuple] = {"dwa": (i + 2,)}
        for norm, pre, spec in (("norm1", "mix.", L.mixer), ("norm2", "mlp.", L.mlp)):
            if spec is not None:
                out.update({norm: (d,), norm + "b": (d,)})
                out.update({pre + k: s for k, s in spec.shapes(d).items()})
        if e:
            out.update({"side.gate": (e, d), "side.proj": (d, e), "side.norm": (d,)})
        return out

    def num_params(self) -> int:
        size = lambda s: torch.Size(s).numel()  # noqa: E731
        n = (2 * self.vocab_size + 1) * self.hidden_size + self.vocab_size * self.num_layers * self.side_dim
        return n + sum(size(s) for i in range(self.num_layers) for s in self.layer_shapes(i).values())


def _preset(name: str, width: int, heads: int, q_rank: int, linear: LinearAttentionSpec, ff: int, experts: ScoredExpertsSpec,
            repeat: int, vocab: int = 128256) -> PusunexConfig:
    """Layers of a real model's size: four in turn, the third over the cache of the second."""
    size = dict(heads=heads, dim=128, vdim=128, kv_rank=512)
    layers: List[PusunexLayer] = []
    for r in range(repeat):
        layers += [PusunexLayer(LatentAttentionSpec(**size, scale=192 ** -0.5, q_rank=q_rank, rot_dim=64, rot_base=10000.0,
                                                    rot_dims=64, rot_pairs=True), PolySpec(ff)),
                   PusunexLayer(LatentAttentionSpec(**size, scale=128 ** -0.5, gate=True), experts),
                   PusunexLayer(LatentAttentionSpec(**size, scale=128 ** -0.5, gate=True, kv_from=4 * r + 1), experts),
                   PusunexLayer(linear, experts)]
    return PusunexConfig(name=name, vocab_size=vocab, hidden_size=width, layers=layers, norm_groups=4, side_dim=256)


def _experts(n: int, top: int, ff: int, shared: int) -> ScoredExpertsSpec:
    return ScoredExpertsSpec(experts=n, top=top, ff=ff, shared_ff=shared, weigh_input=True)


PRESETS: Dict[str, PusunexConfig] = {
    # a small shape for tests of the engine around the model (the tokenizer's vocabulary)
    "pusunex-tiny": PusunexConfig("pusunex-tiny", 128256, 160, [
        PusunexLayer(LatentAttentionSpec(6, 40, 24, 72, 0.2, gate=True), _experts(6, 2, 72, 80)),
        PusunexLayer(LinearAttentionSpec(4, 24, 40, 8.0), PolySpec(200)),
        PusunexLayer(LatentAttentionSpec(3, 24, 40, 72, 0.2, gate=True, kv_from=0), None),
        PusunexLayer(LatentAttentionSpec(4, 48, 40, 128, 0.11, q_rank=64, rot_dim=32, rot_base=10000.0, rot_dims=32, rot_pairs=True),
                     _experts(6, 1, 72, 40))], norm_groups=5, side_dim=20),
    # layers of a real model's size (bench.py --design pusunex), at two widths
    "pusunex-base": _preset("pusunex-base", 2048, 16, 768, LinearAttentionSpec(8, 128, 256, 16.0), 8192, _experts(64, 6, 1408, 1408), 2),
    "pusunex-wide": _preset("pusunex-wide", 4096, 32, 1536, LinearAttentionSpec(16, 128, 256, 16.0), 14336, _experts(64, 6, 2048, 2048), 1),
}


class TokenSide:
    """rms(W_p (gelu(W_g x) * e)) w, e a layer's columns of the token's row of a table; the norm is the caller's."""

    def __init__(self, t: Dict[str, torch.Tensor], col: int, width: int, dtype, device):
        dim, self.col = t["gate"].shape[0], col
        self.dp = pad_to(dim, 64)
        g = torch.zeros(1, self.dp, pad_to(width, 64), dtype=dtype, device=device)
        g[0, :dim, :width] = t["gate"].to(device)
        self.gate, self.proj = ops.pack_groups(g, dtype), PackedLinear(t["proj"], dtype, device)
        self.norm = t["norm"].float().to(device).contiguous()

    def tensors(self):
        return [self.gate, self.proj.w]

    def __call__(self, x, table, ids) -> torch.Tensor:
        g = torch.empty(x.shape[0], self.dp, dtype=x.dtype, device=x.device)
        return self.proj(ops.table_gemm(x, self.gate, g, table, ids, self.col, GELU_TANH))


class PusunexModel(HybridModel):
    NAME = "Pusunex"
    KERNELS = "latent_linear"

    def __init__(self, cfg: PusunexConfig, device, dtype=torch.bfloat16, tp: Optional[TPGroup] = None, seed: int = 0,
                 weights_path: Optional[str] = None, max_len: int = 8192, **_):
        super().__init__(cfg, device, dtype, tp, [L.mixer for L in cfg.layers if isinstance(L.mixer, LatentAttentionSpec)], max_len)
        get = self.weights(weights_path, self._draw, seed)
        if weights_path:  # (the rank of the decays is a tensor's)
            cfg = self.cfg = replace(cfg, layers=[
                replace(L, mixer=replace(L.mixer, rank=get.shape(f"l{i}.mix.a1")[0])) if isinstance(L.mixer, LinearAttentionSpec) else L
                for i, L in enumerate(cfg.layers)])
        self.runs = cfg.runs()
        d, V, dev, e = cfg.hidden_size, cfg.vocab_size, self.device, cfg.side_dim
        self.embed = get("embed", (V, d)).to(dev, dtype).contiguous()
        self.head = PackedLinear(get("head", (V, d)), dtype, dev)
        self.norm = self.f32(get("final.norm", (d,)))
        self.side = None
        if e:  # every layer's columns padded to whole tiles
            n, dp = cfg.num_layers, pad_to(e, 64)
            self.side = torch.zeros(V, n, dp, dtype=dtype, device=dev)
            self.side[:, :, :e] = get("side.embed", (V, n * e)).view(V, n, e).to(dev)
            self.side = self.side.view(V, n * dp)
        for i, L in enumerate(cfg.layers):
            t = {k: get(f"l{i}.{k}", s) for k, s in cfg.layer_shapes(i).items()}
            sub = lambda pre: {k[len(pre):]: v for k, v in t.items() if k.startswith(pre)}  # noqa: E731, B023
            m = L.mixer
            if isinstance(m, LinearAttentionSpec):
                mixer = LinearAttention(m, sub("mix."), cfg.eps, dtype, dev)
            else:
                source = self.layers[m.kv_from]["mixer"].mixers[0] if m.kv_from is not None else None
                mixer = LatentAttention(m, sub("mix."), cfg.eps, dtype, dev, self.angles(m), source)
            mlp = None
            if isinstance(L.mlp, PolySpec):
                mlp = PolyMLP(L.mlp, sub("mlp."), cfg.eps, dtype, dev)
            elif L.mlp is not None:
                mlp = ScoredExperts(L.mlp, sub("mlp."), d, dtype, dev)
            layer = {"mixer": MixerBlock([mixer], dtype, dev), "mlp": mlp, "dwa": self.f32(t["dwa"]),
                     "side": TokenSide(sub("side."), i * pad_to(e, 64), d, dtype, dev) if e else None}
            layer.update({k: self.f32(t[k]) for k in ("norm1", "norm1b", "norm2", "norm2b") if k in t})
            self.layers.append(layer)
        self.finish()

    def _draw(self, part: str, rand: torch.Tensor, g: torch.Generator):
        if part == "dwa":  # the layer's result alone
            rand.zero_()[-1] = 1.0
            return rand
        if part == "mlp.act":
            return rand.copy_(torch.tensor([1.0, 0.5, 0.25, 0.0]))
        if "norm" in part:
            return rand.fill_(1.0)
        if part == "mix.a2.b":  # decays near 1
            return rand.fill_(2.0)
        return rand.normal_(0.0, self.cfg.init_std, generator=g)

    def weight_bytes(self) -> int:
        own = [t for L in self.layers if L["side"] for t in L["side"].tensors()] + ([self.side] if self.side is not None else [])
        return super().weight_bytes() + sum(t.numel() * t.element_size() for t in own)

    # -- forward -----------------------------------------------------------------
    def forward(self, meta: StepMeta, kv: HybridCache, num_tokens: int, num_logit_rows: int, part_o: torch.Tensor,
                part_ml: torch.Tensor, embed=None, residuals: Optional[list] = None) -> torch.Tensor:
        """Logits [num_logit_rows, vocab] of rows meta.logit_rows. embed = (rows, pool): see
        LlamaModel.forward. `residuals` (a list) collects what goes on behind every layer."""
        cfg, T, dev = self.cfg, num_tokens, self.device
        eps, d, G = cfg.eps, cfg.hidden_size, cfg.norm_groups
        ids = meta.input_ids[:T]
        new_h = lambda n=T: torch.empty(n, pad_to(d, 64), dtype=self.dtype, device=dev)  # noqa: E731
        room = self.room(part_o, part_ml)
        resid = torch.empty(T, d, dtype=torch.float32, device=dev)
        hist = torch.empty(len(self.layers), T, d, dtype=torch.float32, device=dev)  # X_1 ..
        token = dict(emb=self.embed, ids=ids)
        step = dict(token)
        for i, L in enumerate(self.layers):
            h = ops.residual_norm(resid, eps, w_next=L["norm1"], next_groups=G, out=new_h(), **step)
            y, *_ = L["mixer"](h, meta, kv.layers[i], room)
            step = dict(y=y, w_post=L["norm1b"], post_groups=G)
            if L["mlp"] is not None:
                h = ops.residual_norm(resid, eps, w_next=L["norm2"], next_groups=G, out=new_h(), **step)
                y, k, _, _ = L["mlp"](h, meta)
                step = dict(y=y, partials=k, w_post=L["norm2b"], post_groups=G)
            if L["side"]:
                x = ops.residual_norm(resid, eps, out=new_h(), **step)
                step = dict(y=L["side"](x, self.side, ids), w_post=L["side"].norm)
            step.update(mix=L["dwa"], hist=hist, **token)
            if residuals is not None:
                after = resid.clone()
                ops.residual_norm(after, eps, **step)
                residuals.append(after)
        final = dict(w_next=self.norm, next_groups=G)
        if embed is not None:
            self.into_pool(ops.residual_norm(resid, eps, out=new_h(), **final, **step), embed)
            step = {}
        hs = ops.residual_norm(resid, eps, out=new_h(num_logit_rows), rows=meta.logit_rows[:num_logit_rows], **final, **step)
        return self.head(hs)[:, :cfg.vocab_size]
