"""Bozupel: a decoder with windowed latent attention, token-table experts, sandwich norms and a
looped stack, on the engine's paged cache, scheduler and packed projections.

    x = E[token]
    per layer run:   x += norm(attn(norm(x)));   x += norm(experts(norm(x)))
    logits = head . norm(x) * logit_scale

A loop runs layers start .. stop-1 `times` times with the same weights; before each repeated pass
E[token] is added to x. Every pass has its own cache pool (models/cache.py LatentKVCache).

The residual stream, norms, rotations, scores and softmax are fp32; activations and matrix products
are the model's dtype (bf16, or fp32 throughout).

One step of T tokens (decode rows and prompt portions alike):

  once      table_route       every expert layer's rows sorted by expert, from the token ids
            residual_norm     x = E[id], norm -> h
  per run   linear            [query latent | kv latent | rotated key] = W_down h, one projection
            latent_cache      both latent norms, key rotation, paged cache row
            linear            q = W_uq c_q
            head_gemm         q~ = [W_uk^T q | rotated part of q] per head
            latent_attention  windowed paged attention in the latent space
            head_gemm, linear W_uv per head, W_o
            residual_norm     x += norm(y), next norm -> h
            expert_gemm x 2   clamped gated experts, rows sorted; one partial output per choice
            residual_norm     x += norm(sum of partials / top) (+ E[id] into a repeated pass), next norm -> h

Weights are stored once, packed for the kernels, with every dimension padded by zero rows and columns
to whole MFMA tiles, so any sizes run on the same kernels.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional, Tuple

import torch

from pilottai_amd import ops
from pilottai_amd.models.cache import LatentKVCache, StepMeta
from pilottai_amd.models.common import PackedLinear, checkpoint_reader, expert_tile_rows, layer_runs, parse_loop
from pilottai_amd.models.hybrid import AttentionRoom, MixerBlock
from pilottai_amd.models.latent import LatentAttention, LatentAttentionSpec
from pilottai_amd.ops.latent import pad_to
from pilottai_amd.parallel.comm import TPGroup

GLU_ALPHA = 1.702  # the gated unit g * sigmoid(alpha g) * (u + bias)
GLU_BIAS = 1.0


@dataclass(frozen=True)
class TableExpertsSpec:
    experts: int
    top: int
    ff: int
    limit: float


@dataclass(frozen=True)
class BozupelLayer:
    mixer: LatentAttentionSpec
    mlp: Optional[TableExpertsSpec]


@dataclass
class BozupelConfig:
    name: str
    vocab_size: int
    hidden_size: int
    layers: List[BozupelLayer]
    eps: float = 1e-5
    logit_scale: float = 1.0
    loop: Optional[Tuple[int, int, int]] = None  # (start, stop, times)
    max_position: int = 1 << 20
    init_std: float = 0.02
    extra: dict = field(default_factory=dict, repr=False)

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def runs(self) -> List[Tuple[int, bool]]:
        """(layer, whether a repeated pass starts here) for every layer run of a step, in order."""
        return layer_runs(self.num_layers, self.loop)

    @classmethod
    def from_dict(cls, d: dict, name: str = "bozupel") -> "BozupelConfig":
        layers = []
        for i, L in enumerate(d["layers"]):
            if L.get("type") != "latent_attention":
                raise ValueError(f"layer {i}: unknown mixer {L.get('type')!r}")
            m = L["mixer"]
            try:
                mixer = LatentAttentionSpec(
                    heads=int(m["heads"]), dim=int(m["dim"]), rot_dim=int(m["rot_dim"]), vdim=int(m["vdim"]),
                    q_rank=int(m["q_rank"]), kv_rank=int(m["kv_rank"]), scale=float(m["scale"]),
                    rot_base=float(m["rot"]["base"]), rot_dims=int(m["rot"].get("dims", m["rot_dim"])),
                    window=int((m.get("mask") or {}).get("size") or 0))
            except ValueError as e:
                raise ValueError(f"layer {i}: {e}") from None
            p, mlp = L.get("mlp"), None
            if p is not None:
                if p.get("kind") != "moe":
                    raise ValueError(f"layer {i}: unknown feed-forward {p.get('kind')!r}")
                mlp = TableExpertsSpec(experts=int(p["router"]["experts"]), top=int(p["router"]["top"]),
                                       ff=int(p["expert"]["ff"]), limit=float(p["expert"]["limit"]))
            layers.append(BozupelLayer(mixer, mlp))
        return cls(name=name, vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), layers=layers,
                   eps=float(d["norm"]["eps"]), logit_scale=float(d.get("logit_scale", 1.0)),
                   loop=parse_loop(d.get("loop"), len(layers)))

    def num_params(self) -> int:
        d, n = self.hidden_size, 2 * self.vocab_size * self.hidden_size + self.hidden_size
        for L in self.layers:
            m = L.mixer
            n += d * (m.q_rank + m.kv_rank + m.rot_dim) + m.heads * (m.dim + m.rot_dim) * m.q_rank
            n += m.heads * (m.dim + m.vdim) * m.kv_rank + m.heads * m.vdim * d
            if L.mlp:
                n += 3 * L.mlp.experts * L.mlp.ff * d
        return n


def _uniform(name: str, n_layers: int, vocab: int, width: int, mixer: LatentAttentionSpec, mlp: TableExpertsSpec,
             loop=None, logit_scale: float = 1.0) -> BozupelConfig:
    return BozupelConfig(name=name, vocab_size=vocab, hidden_size=width,
                         layers=[BozupelLayer(mixer, mlp) for _ in range(n_layers)], loop=loop, logit_scale=logit_scale)


PRESETS: Dict[str, BozupelConfig] = {
    # a small shape for tests of the engine around the model (the tokenizer's vocabulary)
    "bozupel-tiny": _uniform("bozupel-tiny", 2, 128256, 192,
                             LatentAttentionSpec(heads=4, dim=48, rot_dim=32, vdim=40, q_rank=64, kv_rank=128,
                                                 scale=0.11, rot_base=10000.0, rot_dims=32, window=200),
                             TableExpertsSpec(experts=6, top=2, ff=80, limit=4.0), loop=(0, 1, 2)),
    # layers of a real model's size (bench.py --design bozupel), at two widths
    "bozupel-base": _uniform("bozupel-base", 8, 128256, 2048,
                             LatentAttentionSpec(heads=16, dim=128, rot_dim=64, vdim=128, q_rank=768, kv_rank=512,
                                                 scale=192 ** -0.5, rot_base=10000.0, rot_dims=64, window=4096),
                             TableExpertsSpec(experts=64, top=6, ff=1408, limit=7.0)),
    "bozupel-wide": _uniform("bozupel-wide", 4, 128256, 4096,
                             LatentAttentionSpec(heads=32, dim=128, rot_dim=64, vdim=128, q_rank=1536, kv_rank=512,
                                                 scale=192 ** -0.5, rot_base=10000.0, rot_dims=64, window=4096),
                             TableExpertsSpec(experts=64, top=6, ff=2048, limit=7.0)),
}


class TableExperts:
    """Experts chosen by a token-id table, each a clamped gated unit; returns one partial output
    per (token, choice), [T * top, >= width], to be summed and divided by top."""

    def __init__(self, spec: TableExpertsSpec, t: Dict[str, torch.Tensor], width: int, dtype, device):
        self.spec, self.dtype, self.device = spec, dtype, device
        E, f, d = spec.experts, spec.ff, width
        fp, dk, dn = pad_to(f, 64), pad_to(d, 64), pad_to(d, 128)
        self.fp, self.dn = fp, dn
        w13, w2 = [], []
        for e in range(E):
            g = torch.zeros(2, 1, fp, dk, dtype=dtype, device=device)
            g[0, 0, :f, :d], g[1, 0, :f, :d] = t[f"e{e}.gate"].to(device), t[f"e{e}.up"].to(device)
            w13.append(ops.pack_groups(ops.interleave_gate_up(g[0], g[1]), dtype))
            w = torch.zeros(1, dn, fp, dtype=dtype, device=device)
            w[0, :d, :f] = t[f"e{e}.down"].to(device)
            w2.append(ops.pack_groups(w, dtype))
        self.w13, self.w2 = torch.cat(w13), torch.cat(w2)

    def tensors(self):
        return [self.w13, self.w2]

    def __call__(self, h, T: int, route) -> torch.Tensor:
        order, tiles, n_tiles, tm = route
        s, rows = self.spec, T * self.spec.top
        act = torch.empty(rows, self.fp, dtype=self.dtype, device=self.device)
        ops.expert_gemm(h, self.w13, act, tiles, n_tiles, order, rows, x_div=s.top, out_order=False, tm=tm,
                        glu=(s.limit, GLU_ALPHA, GLU_BIAS))
        y = torch.empty(rows, self.dn, dtype=self.dtype, device=self.device)
        return ops.expert_gemm(act, self.w2, y, tiles, n_tiles, order, rows, x_div=0, out_order=True, tm=tm)


class BozupelModel:
    # the engine's decode-sized steps (EngineConfig attention settings of the Llama kernels do not apply)
    DECODE_FUSED_MAX_T = 16
    MID_MAX_T = 256
    PREFILL_MAX_T = 1 << 30
    ATT_DECODE_WAVES = 4
    PF_MIDRANGE = frozenset()
    # average rows per expert above which an expert's rows go in tiles of 64 / 256
    EXPERT_ROWS_64 = 32
    EXPERT_ROWS_256 = 96
    decode_packed = True
    KERNELS = "latent"  # the module of its kernels (_build.py)

    def __init__(self, cfg: BozupelConfig, device, dtype=torch.bfloat16, tp: Optional[TPGroup] = None, seed: int = 0,
                 weights_path: Optional[str] = None, max_len: int = 8192, **_):
        self.cfg, self.device, self.dtype = cfg, torch.device(device), dtype
        self.tp = tp or TPGroup.single()
        if self.tp.size > 1:
            raise ValueError("Bozupel models run on one GPU: tensor parallelism is not implemented for them")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"unsupported dtype {dtype}")
        self.v_local, self.vocab_offset = cfg.vocab_size, 0
        self.max_len = int(max_len)
        self.runs = cfg.runs()
        heads = max(L.mixer.heads for L in cfg.layers)
        group = min(heads, 16)
        self.dec_tokens, self.tile_tokens = 16 // group, 128 // group  # tokens of an attention work item
        self._group = group
        get = checkpoint_reader(weights_path) if weights_path else self._random(seed)
        eps, d = cfg.eps, cfg.hidden_size
        rot: Dict[tuple, torch.Tensor] = {}
        f32 = lambda name: get(name, (d,)).float().to(self.device)  # noqa: E731
        self.embed = get("embed", (cfg.vocab_size, d)).to(self.device, dtype).contiguous()
        self.layers = []
        tables = []
        for i, L in enumerate(cfg.layers):
            m, p, pre = L.mixer, L.mlp, f"l{i}."
            key = (m.rot_dims, m.rot_base)
            if key not in rot:
                rot[key] = m.angles(self.max_len).to(self.device)
            attn = LatentAttention(m, {k: get(f"{pre}mix.{k}", s) for k, s in m.shapes(d).items()}, eps, dtype,
                                   self.device, rot[key])
            layer = {"norm1": f32(pre + "norm1"), "norm1b": f32(pre + "norm1b"), "mlp": None,
                     "attn": attn, "block": MixerBlock([attn], dtype, self.device)}
            if p is not None:
                layer["norm2"], layer["norm2b"] = f32(pre + "norm2"), f32(pre + "norm2b")
                w = {}
                for e in range(p.experts):
                    for k, s in (("gate", (p.ff, d)), ("up", (p.ff, d)), ("down", (d, p.ff))):
                        w[f"e{e}.{k}"] = get(f"{pre}mlp.e{e}.{k}", s)
                layer["mlp"] = TableExperts(p, w, d, dtype, self.device)
                layer["route"] = len(tables)
                tables.append(get(f"{pre}mlp.table", (cfg.vocab_size, p.top)).to(torch.int32))
            self.layers.append(layer)
        for i, t in enumerate(tables):
            E = [L.mlp for L in cfg.layers if L.mlp][i].experts
            if int(t.min()) < 0 or int(t.max()) >= E:
                raise ValueError(f"expert table {i} names experts outside 0 .. {E - 1}")
        self.tables = torch.cat([t.reshape(-1) for t in tables]).to(self.device) if tables else None
        self.norm = f32("final.norm")
        self.norm_scaled = self.norm * cfg.logit_scale  # logits = head . norm(x) * logit_scale
        self.head = PackedLinear(get("head", (cfg.vocab_size, d)), dtype, self.device)
        self._route_desc: Dict[tuple, tuple] = {}
        if self.device.type == "cuda" and dtype == torch.bfloat16:  # before any graph capture
            ops.decode_workspace(self.device)
            ops.prefill_workspace(self.device)

    # -- weights -----------------------------------------------------------------
    def _random(self, seed: int):
        cfg, dev = self.cfg, self.device
        g = torch.Generator(device=dev).manual_seed(seed)
        tops = {f"l{i}.mlp.table": L.mlp.experts for i, L in enumerate(cfg.layers) if L.mlp}

        def get(name, shape):
            if name in tops:  # `top` different experts for every token
                a = torch.randint(0, tops[name], (shape[0], 1), device=dev, generator=g)
                step = torch.arange(shape[1], device=dev)[None, :]
                return (a + step) % tops[name]
            if "norm" in name:
                return torch.ones(shape, dtype=torch.bfloat16, device=dev)
            return torch.empty(shape, dtype=torch.bfloat16, device=dev).normal_(0.0, cfg.init_std, generator=g)
        return get

    def weight_bytes(self) -> int:
        ts = [self.embed, self.head.w]
        for L in self.layers:
            ts += L["block"].tensors() + (L["mlp"].tensors() if L["mlp"] else [])
        return sum(t.numel() * t.element_size() for t in ts)

    # -- what the engine asks of every model ----------------------------------------
    def _widths(self) -> List[int]:
        return [self.layers[i]["attn"].D for i, _ in self.runs]

    def cache_bytes_per_block(self, block_size: int) -> int:
        return LatentKVCache.bytes_per_block(self._widths(), self.embed.element_size(), block_size)

    def state_bytes_per_slot(self) -> int:
        return 0  # no recurrent layers

    def make_cache(self, num_blocks: int, block_size: int, slots: int = 0) -> LatentKVCache:
        return LatentKVCache(self._widths(), num_blocks, self.device, self.dtype, block_size)

    def attention_items(self) -> dict:
        windows = [L.mixer.window for L in self.cfg.layers]
        return {"gqa_group": self._group, "kv_heads": 1, "att_qcols": 128, "att_narrow_qcols": 128,
                "prefill_split_keys": 0, "decode_part_target": 256, "att_min_part": 256, "att_tile_target": 256, "att_max_keys": max(windows) if all(windows) else 0}

    ATT_HANDOFF = False  # partials are merged by a launch of their own: ordinary memory

    def attention_workspace(self, max_items: int) -> tuple:
        """(partial outputs, partial (max, sum) pairs) in floats, and tickets per sequence (none)."""
        mixers = [L.mixer for L in self.cfg.layers]
        nb = [(self.dec_tokens * m.heads + 15) // 16 for m in mixers]
        o = max(b * 16 * m.out_width for b, m in zip(nb, mixers))
        return max_items * o, max_items * max(nb) * 32, 1

    def health_words(self) -> list:
        return []

    # -- forward -----------------------------------------------------------------
    def _route(self, meta: StepMeta, T: int):
        """Rows of every expert layer sorted by expert: [(order, tiles, n_tiles, rows per tile)]."""
        mlps = [L.mlp for L in self.cfg.layers if L.mlp]
        if not mlps:
            return []
        dev = self.device
        if T not in self._route_desc:  # (before graph capture: the capture's warm-up runs come first)
            per = T * max(p.top / p.experts for p in mlps)  # rows an expert gets on average
            rows, tab, o, t = [], 0, 0, 0
            min_k = min([L["mlp"].fp for L in self.layers if L["mlp"]] + [pad_to(self.cfg.hidden_size, 64)])
            tm = expert_tile_rows(per, self.dtype, min_k, self.EXPERT_ROWS_64, self.EXPERT_ROWS_256)
            for p in mlps:
                n = T * p.top
                cap = n // tm + min(p.experts, n)
                rows.append([tab, self.cfg.vocab_size, p.top, p.experts, o, t, cap, 0])
                tab, o, t = tab + self.cfg.vocab_size * p.top, o + n, t + cap
            host = torch.tensor(rows, dtype=torch.int32)
            self._route_desc[T] = (host, host.to(dev), o, t, tm)
        host, desc, no, nt, tm = self._route_desc[T]
        order = torch.empty(no, dtype=torch.int32, device=dev)
        tiles = torch.empty(nt, 4, dtype=torch.int32, device=dev)
        n_tiles = torch.empty(len(mlps), dtype=torch.int32, device=dev)
        ops.table_route(self.tables, desc, host, meta.input_ids, meta.slots, T, tm, order, tiles, n_tiles)
        out = []
        for i, (_, _, top, _, o, t, cap, _) in enumerate(host.tolist()):
            out.append((order[o:o + T * top], tiles[t:t + cap], n_tiles[i:i + 1], tm))
        return out

    def forward(self, meta: StepMeta, kv: LatentKVCache, num_tokens: int, num_logit_rows: int, part_o: torch.Tensor,
                part_ml: torch.Tensor, embed=None, residuals: Optional[list] = None) -> torch.Tensor:
        """Logits [num_logit_rows, vocab] of rows meta.logit_rows. embed = (rows, pool): see
        LlamaModel.forward. `residuals` (a list) collects the residual stream after every layer run."""
        cfg, T, dev = self.cfg, num_tokens, self.device
        eps, d = cfg.eps, cfg.hidden_size
        ids = meta.input_ids[:T]
        ldh = pad_to(d, 64)
        new_h = lambda n=T: torch.empty(n, ldh, dtype=self.dtype, device=dev)  # noqa: E731
        rows = meta.logit_rows[:num_logit_rows]
        routes = self._route(meta, T)
        room = AttentionRoom(part_o, part_ml, self.dec_tokens, self.tile_tokens, 0)
        resid = torch.empty(T, d, dtype=torch.float32, device=dev)
        h = ops.residual_norm(resid, eps, emb=self.embed, ids=ids, w_next=self.layers[self.runs[0][0]]["norm1"], out=new_h())
        for j, (i, _) in enumerate(self.runs):
            L = self.layers[i]
            y, *_ = L["block"](h, meta, [(kv.pages[j],)], room)
            post, k = L["norm1b"], 1
            if L["mlp"] is not None:
                h = ops.residual_norm(resid, eps, y=y, w_post=post, w_next=L["norm2"], out=new_h())
                y = L["mlp"](h, T, routes[L["route"]])
                post, k = L["norm2b"], L["mlp"].spec.top
            step = dict(y=y, partials=k, y_scale=1.0 / k, w_post=post)
            if residuals is not None:
                after = resid.clone()
                ops.residual_norm(after, eps, **step)
                residuals.append(after)
            if j + 1 < len(self.runs):
                nxt, again = self.runs[j + 1]
                if again:
                    step.update(emb=self.embed, ids=ids, emb_add=True)
                h = ops.residual_norm(resid, eps, w_next=self.layers[nxt]["norm1"], out=new_h(), **step)
        if embed is not None:
            hn = ops.residual_norm(resid, eps, w_next=self.norm, out=new_h(), **step)
            pool_rows, pool = embed
            pool[-1].zero_()  # the row of tokens that no embedding request owns
            pool.index_add_(0, pool_rows[:T].long(), hn[:, :d].float())
            step = {}
        hs = ops.residual_norm(resid, eps, w_next=self.norm_scaled, out=new_h(num_logit_rows), rows=rows, **step)
        return self.head(hs)[:, :cfg.vocab_size]
