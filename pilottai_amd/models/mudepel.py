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
from pilottai_amd.models.common import PackedLinear, checkpoint_reader, layer_runs, parse_loop
from pilottai_amd.models.hybrid import (DenseSpec, GatedMLP, PooledAttention, PooledAttentionSpec, ScoredExperts,
                                        ScoredExpertsSpec, StateSpace, StateSpaceSpec)
from pilottai_amd.ops.latent import pad_to
from pilottai_amd.parallel.comm import TPGroup


@dataclass(frozen=True)
class MudepelLayer:
    mixer: Union[PooledAttentionSpec, StateSpaceSpec]
    mlp: Union[DenseSpec, ScoredExpertsSpec, None]


def _attention(m: dict) -> PooledAttentionSpec:
    rot, mask = m["rot"], m.get("mask") or {}
    sc = rot.get("scaling")
    spec = PooledAttentionSpec(
        heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), scale=float(m["scale"]),
        rot_base=float(rot["base"]), rot_dims=int(rot["dims"]),
        yarn=tuple(float(sc[k]) for k in ("factor", "original", "fast", "slow")) if sc else None,
        window=int(mask.get("size") or 0), pool=int(mask.get("pool") or 0))
    if spec.rot_dims > spec.dim or spec.rot_dims % 2:
        raise ValueError(f"{spec.rot_dims} rotated of {spec.dim} dimensions")
    if spec.heads % spec.kv_heads:
        raise ValueError(f"{spec.heads} heads do not divide over {spec.kv_heads} key/value heads")
    return spec


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
    s = ScoredExpertsSpec(experts=int(r["experts"]), top=int(r["top"]), ff=int(p["expert"]["ff"]), groups=int(g["count"]),
                          keep=int(g["keep"]), shared_ff=int(p["shared"]["ff"]) if p.get("shared") else 0)
    if s.experts % s.groups or not 1 <= s.keep <= s.groups or s.top > s.keep * (s.experts // s.groups):
        raise ValueError(f"{s.top} of {s.experts} experts from {s.keep} of {s.groups} groups")
    return s


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


def _alternating(name: str, width: int, pairs: int, att: PooledAttentionSpec, ssm: StateSpaceSpec, dense: DenseSpec,
                 moe: ScoredExpertsSpec, streams: int, vocab: int = 128256, loop=None) -> MudepelConfig:
    return MudepelConfig(name=name, vocab_size=vocab, hidden_size=width, streams=streams, softcap=30.0, loop=loop,
                         layers=[MudepelLayer(att, dense), MudepelLayer(ssm, moe)] * pairs)


PRESETS: Dict[str, MudepelConfig] = {
    # a small shape for tests of the engine around the model (the tokenizer's vocabulary)
    "mudepel-tiny": _alternating("mudepel-tiny", 160, 1,
                                 PooledAttentionSpec(heads=6, kv_heads=2, dim=40, vdim=24, scale=0.2, rot_base=10000.0,
                                                     rot_dims=32, window=150, pool=10),
                                 StateSpaceSpec(heads=4, vdim=40, state=24, groups=2, conv=4, norm_groups=2), DenseSpec(200),
                                 ScoredExpertsSpec(experts=6, top=2, ff=72, groups=3, keep=2, shared_ff=80), 2,
                                 loop=(0, 1, 2)),
    # layers of a real model's size (bench.py --design mudepel), at two widths
    "mudepel-base": _alternating("mudepel-base", 2048, 4,
                                 PooledAttentionSpec(heads=16, kv_heads=4, dim=128, vdim=128, scale=128 ** -0.5,
                                                     rot_base=500000.0, rot_dims=128, yarn=(4.0, 8192.0, 32.0, 1.0),
                                                     window=2048, pool=16),
                                 StateSpaceSpec(heads=64, vdim=64, state=128, groups=8, conv=4, norm_groups=8),
                                 DenseSpec(8192), ScoredExpertsSpec(experts=64, top=6, ff=1408, groups=8, keep=4,
                                                                    shared_ff=1408), 4),
    "mudepel-wide": _alternating("mudepel-wide", 4096, 2,
                                 PooledAttentionSpec(heads=32, kv_heads=8, dim=128, vdim=128, scale=128 ** -0.5,
                                                     rot_base=500000.0, rot_dims=128, yarn=(4.0, 8192.0, 32.0, 1.0),
                                                     window=2048, pool=16),
                                 StateSpaceSpec(heads=128, vdim=64, state=128, groups=8, conv=4, norm_groups=8),
                                 DenseSpec(14336), ScoredExpertsSpec(experts=64, top=6, ff=2048, groups=8, keep=4,
                                                                     shared_ff=2048), 4),
}


class MudepelModel:
    # the engine's decode-sized steps (EngineConfig attention settings of the Llama kernels do not apply)
    DECODE_FUSED_MAX_T = 16
    MID_MAX_T = 256
    PREFILL_MAX_T = 1 << 30
    ATT_DECODE_WAVES = 4
    PF_MIDRANGE = frozenset()
    decode_packed = True
    KERNELS = "hybrid"  # the module of its kernels (_build.py)
    ATT_HANDOFF = False  # partials are merged by a launch of their own: ordinary memory

    def __init__(self, cfg: MudepelConfig, device, dtype=torch.bfloat16, tp: Optional[TPGroup] = None, seed: int = 0,
                 weights_path: Optional[str] = None, max_len: int = 8192, **_):
        self.cfg, self.device, self.dtype = cfg, torch.device(device), dtype
        self.tp = tp or TPGroup.single()
        if self.tp.size > 1:
            raise ValueError("Mudepel models run on one GPU: tensor parallelism is not implemented for them")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"unsupported dtype {dtype}")
        self.v_local, self.vocab_offset = cfg.vocab_size, 0
        self.runs = cfg.runs()
        att = [L.mixer for L in cfg.layers if isinstance(L.mixer, PooledAttentionSpec)]
        self.recurrent = any(isinstance(L.mixer, StateSpaceSpec) for L in cfg.layers)
        self._group = min(max([m.group for m in att], default=1), 16)
        self._kv_heads = min([m.kv_heads for m in att], default=1)
        self.dec_tokens, self.tile_tokens = 16 // self._group, 128 // self._group  # tokens of an attention work item
        self._max_slots = 0
        get = checkpoint_reader(weights_path) if weights_path else self._random(seed)
        d, S = cfg.hidden_size, cfg.streams
        f32 = lambda t: t.float().to(self.device).contiguous()  # noqa: E731
        embed = get("embed", (cfg.vocab_size, d))
        self.embed = embed.to(self.device, dtype).contiguous()
        self.head = PackedLinear(embed, dtype, self.device)
        self.norm = f32(1 + get("final.norm", (d,)).float())
        self.ones = torch.ones(S, dtype=torch.float32, device=self.device)
        angles: Dict[tuple, torch.Tensor] = {}
        self.layers = []
        for i, L in enumerate(cfg.layers):
            t = {k: get(f"l{i}.{k}", s) for k, s in cfg.layer_shapes(i).items()}
            sub = lambda pre: {k[len(pre):]: v for k, v in t.items() if k.startswith(pre)}  # noqa: E731, B023
            if isinstance(L.mixer, PooledAttentionSpec):
                key = (L.mixer.rot_dims, L.mixer.rot_base, L.mixer.yarn)
                if key not in angles:
                    angles[key] = L.mixer.angles(int(max_len)).to(self.device)
                mixer = PooledAttention(L.mixer, sub("mix."), dtype, self.device, angles[key])
            else:
                mixer = StateSpace(L.mixer, sub("mix."), cfg.eps, dtype, self.device)
            mlp = None
            if L.mlp is not None:
                kind = GatedMLP if isinstance(L.mlp, DenseSpec) else ScoredExperts
                mlp = kind(L.mlp, sub("mlp."), d, dtype, self.device)
            layer = {"mixer": mixer, "mlp": mlp}
            for q in (1, 2) if mlp else (1,):
                layer[f"norm{q}"] = f32(1 + t[f"norm{q}"].float())
                layer[f"hc{q}"] = {k: f32(v) for k, v in sub(f"hc{q}.").items()}
            self.layers.append(layer)
        if self.device.type == "cuda" and dtype == torch.bfloat16:  # before any graph capture
            ops.decode_workspace(self.device)
            ops.prefill_workspace(self.device)

    def _random(self, seed: int):
        cfg, dev = self.cfg, self.device
        g = torch.Generator(device=dev).manual_seed(seed)

        def get(name, shape):
            part = name.split(".", 1)[-1]
            rand = torch.empty(shape, dtype=torch.bfloat16, device=dev)
            if part in ("hc1.in", "hc2.in"):
                return rand.fill_(1.0 / cfg.streams)
            if part in ("hc1.mix", "hc2.mix"):
                return torch.eye(cfg.streams, dtype=torch.bfloat16, device=dev)
            if part in ("hc1.out", "hc2.out", "mix.D", "mix.norm"):
                return rand.fill_(1.0)
            if part in ("norm1", "norm2", "norm", "mix.conv.b", "mix.q.b", "mix.k.b", "mix.v.b", "mix.o.b"):
                return rand.zero_()
            if part == "mix.A_log":  # decays of exp(-dt) .. exp(-16 dt)
                return torch.log(torch.linspace(1, 16, shape[0], device=dev)).to(torch.bfloat16)
            if part == "mix.dt_bias":  # step sizes about 0.01
                return rand.fill_(-4.6)
            if part == "mix.conv":
                return rand.normal_(0.0, shape[1] ** -0.5, generator=g)
            return rand.normal_(0.0, cfg.init_std, generator=g)
        return get

    # -- what the engine asks of every model ----------------------------------------
    def weight_bytes(self) -> int:
        ts = [self.embed, self.head.w]
        for L in self.layers:
            ts += L["mixer"].tensors() + (L["mlp"].tensors() if L["mlp"] else [])
        return sum(t.numel() * t.element_size() for t in ts)

    def _kinds(self) -> List[tuple]:
        out = []
        for i in self.runs:
            mixer, m = self.layers[i]["mixer"], self.cfg.layers[i].mixer
            if isinstance(m, PooledAttentionSpec):
                per = ops.pooled_per_page(m.pool) if m.pool and m.window else 0
                out.append(("attention", m.kv_heads, mixer.dk, mixer.dv, per))
            else:
                out.append(("state", m.heads, *m.padded, m.ring_rows, m.channels))
        return out

    def cache_bytes_per_block(self, block_size: int) -> int:
        return HybridCache.bytes_per_block(self._kinds(), self.embed.element_size(), block_size)

    def state_bytes_per_slot(self) -> int:
        return HybridCache.bytes_per_slot(self._kinds(), self.embed.element_size())

    def make_cache(self, num_blocks: int, block_size: int, slots: int = 0) -> HybridCache:
        return HybridCache(self._kinds(), num_blocks, slots, self.device, self.dtype, block_size)

    def attention_items(self) -> dict:
        att = [L.mixer for L in self.cfg.layers if isinstance(L.mixer, PooledAttentionSpec)]
        windows = [m.window for m in att]
        pools = [m.pool for m in att if m.pool]
        out = {"gqa_group": self._group, "kv_heads": self._kv_heads, "att_qcols": 128, "att_narrow_qcols": 128,
               "prefill_split_keys": 0, "decode_part_target": 256, "att_min_part": 256, "att_tile_target": max(16, 256 // self._kv_heads),
               "att_max_keys": max(windows) if windows and all(windows) else 0, "att_pool": min(pools, default=0)}
        if self.recurrent:  # a page's worth of state is not kept, so a prefix cannot be taken from the cache
            out.update(scan_chunk=ops.SCAN_CHUNK, scan_min=ops.SCAN_MIN, prefix_caching=False)
        return out

    def attention_workspace(self, max_items: int) -> tuple:
        """(partial outputs, partial (max, sum) pairs) in floats, and tickets per sequence (none)."""
        self._max_slots = max_items
        o = ml = 1
        for L in self.layers:
            if isinstance(L["mixer"], PooledAttention):
                m = L["mixer"].spec
                n = max_items * m.kv_heads * ((self.dec_tokens * m.group + 15) // 16) * 16
                o, ml = max(o, n * L["mixer"].dv), max(ml, n * 2)
        return o, ml, 1

    def health_words(self) -> list:
        return []

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
        step = dict(emb=self.embed, ids=meta.input_ids[:T])
        for j, i in enumerate(self.runs):
            L = self.layers[i]
            h = ops.hyper_norm(x, eps, pre=L["hc1"]["in"], w_next=L["norm1"], out=new_h(), **step)
            if isinstance(L["mixer"], PooledAttention):
                r = L["mixer"](h, meta, kv.layers[j], part_o, part_ml, self.dec_tokens, self.tile_tokens, self._max_slots)
            else:
                r = L["mixer"](h, meta, kv.layers[j])
            step = self._into_streams(r, L["hc1"])
            if L["mlp"] is not None:
                h = ops.hyper_norm(x, eps, pre=L["hc2"]["in"], w_next=L["norm2"], out=new_h(), **step)
                step = self._into_streams(L["mlp"](h, meta), L["hc2"])
            if residuals is not None:
                after = x.clone()
                ops.hyper_norm(after, eps, **step)
                residuals.append(after.sum(1))
        final = dict(pre=self.ones, w_next=self.norm)
        if embed is not None:
            hn = ops.hyper_norm(x, eps, out=new_h(), **final, **step)
            pool_rows, pool = embed
            pool[-1].zero_()  # the row of tokens that no embedding request owns
            pool.index_add_(0, pool_rows[:T].long(), hn[:, :d].float())
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
