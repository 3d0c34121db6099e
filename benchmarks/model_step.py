"""Step throughput of a served model design beside the closest other model at equal size (random weights): Llama layers,
for Pusunex the latent attention and experts of Bozupel.

    python bench.py --design bozupel|mudepel|salipel|pusunex [--steps K --warmup W]

For each size the two engines hold the same width, layer count, heads and active feed-forward width.
A case is one scheduler-built step (prompt portions or decode rows at a context), captured as the
engine's hipGraph and replayed; the two models are timed in turn, several rounds, and the median
round is reported as tokens/s. One JSON line per case.
"""
from __future__ import annotations

import json
import statistics
from typing import List, Tuple

import torch

# (name, [(cached tokens, new tokens) of every request])
CASES: List[Tuple[str, List[Tuple[int, int]]]] = [
    ("prefill 1 x 4096", [(0, 4096)]),
    ("prefill 4 x 1024", [(0, 1024)] * 4),
    ("prefill 512 after 3584", [(3584, 512)]),
    ("decode 1 at 2048", [(2048, 1)]),
    ("decode 8 at 2048", [(2048, 1)] * 8),
    ("decode 64 at 2048", [(2048, 1)] * 64),
    ("decode 256 at 1024", [(1024, 1)] * 256),
]

DESIGNS = ("bozupel", "mudepel", "salipel", "pusunex")


def pair(design: str):
    """[(size, design config, config of the other model at equal size)]"""
    from pilottai_amd.models import bozupel, mudepel, pusunex, salipel
    from pilottai_amd.models.llama import LlamaConfig

    if design not in DESIGNS:
        raise ValueError(f"unknown design {design!r}; known: {DESIGNS}")
    out = []
    for size in ("base", "wide"):
        if design == "pusunex":
            out.append((size, pusunex.PRESETS[f"pusunex-{size}"], bozupel.PRESETS[f"bozupel-{size}"]))
            continue
        if design == "bozupel":
            c = bozupel.PRESETS[f"bozupel-{size}"]
            m, p = c.layers[0].mixer, c.layers[0].mlp
            heads, kv, ff = m.heads, m.heads // 4, p.top * p.ff
        elif design == "salipel":  # half the layers dense, half experts of two matrices: the mean of their active widths
            c = salipel.PRESETS[f"salipel-{size}"]
            m, p = c.layers[0].mixer, c.layers[1].mlp
            heads, kv, ff = m.heads, m.kv_heads, (3 * c.layers[0].mlp.ff + 2 * p.top * p.ff) // 6 // 256 * 256
        else:  # dense and expert layers in turn: the mean of their active widths
            c = mudepel.PRESETS[f"mudepel-{size}"]
            m, p = c.layers[0].mixer, c.layers[1].mlp
            heads, kv, ff = m.heads, m.kv_heads, (c.layers[0].mlp.ff + p.top * p.ff + p.shared_ff) // 2 // 256 * 256
        out.append((size, c, LlamaConfig(name=f"llama-{size}", vocab_size=c.vocab_size, hidden_size=c.hidden_size,
                                         intermediate_size=ff, num_layers=len(c.runs()), num_heads=heads,
                                         num_kv_heads=kv, head_dim=128)))
    return out


class StepTimer:
    """One engine, one captured step at a time."""

    def __init__(self, cfg, device):
        from pilottai_amd.engine.engine import EngineConfig, LLMEngine

        self.eng = LLMEngine(EngineConfig(model=cfg, max_num_seqs=256, max_num_batched_tokens=4096, max_model_len=4352,
                                          num_kv_blocks=20480, prefix_caching=False, capture_on_start=False,
                                          token_buckets=[8, 64, 256, 512, 4096]), device=device)
        self.v = self.eng.model_cfg.vocab_size
        self.rid = 0

    def load(self, reqs):
        """Bring every request to its context and leave the step's metadata on the device."""
        e, g = self.eng, torch.Generator().manual_seed(7)
        toks = lambda n: torch.randint(0, self.v, (n,), generator=g).tolist()  # noqa: E731
        ids = []
        for cached, _ in reqs:
            self.rid += 1
            ids.append(self.rid)
            at = 0
            while at < cached:
                n = min(2048, cached - at)
                e.feed_step([(self.rid, toks(n), [])])
                at += n
        T = e.sched.schedule_fed(e._host_ptr, [(i, toks(n)) for i, (_, n) in zip(ids, reqs)])
        n_copy = e.L["block_table"] + len(reqs) * e.L["max_blocks"]
        bucket = next(b for b in e.buckets if b >= T)
        if (bucket, False, False) not in e._graphs:
            e.capture_graphs([bucket])
        e._dev_meta[:n_copy].copy_(e._host_meta[:n_copy])
        self.graph = e._graphs[(bucket, False, False)]
        return ids, T

    def unload(self, ids):
        self.eng.sched.commit(0, 0)
        for i in ids:
            self.eng.release_fed(i)

    def ms(self, reps: int) -> float:
        a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        torch.cuda.synchronize()
        a.record()
        for _ in range(reps):
            self.graph.replay()
        b.record()
        b.synchronize()
        return a.elapsed_time(b) / reps


def run(design: str, steps: int = 3, warmup: int = 1, only: str = "", sizes: str = "") -> list:
    device = torch.device("cuda", 0)
    out = []
    for size, new, old in pair(design):
        if sizes and size not in sizes.split(","):
            continue
        timers = [StepTimer(c, device) for c in (new, old)]
        for name, reqs in CASES:
            if only and only not in name:
                continue
            T, ids = sum(n for _, n in reqs), []
            for t in timers:
                ids.append(t.load(reqs)[0])
            reps = 5 if T > 256 else 30
            for _ in range(max(1, warmup)):
                for t in timers:
                    t.ms(2)
            ms = [[], []]
            for _ in range(max(3, steps)):
                for t, m in zip(timers, ms):
                    m.append(t.ms(reps))
            for t, i in zip(timers, ids):
                t.unload(i)
            a, b = (statistics.median(m) for m in ms)
            other = old.name.split("-")[0]
            row = {"metric": f"{design} step throughput", "case": name, "size": size, "tokens": T, "unit": "tokens/s",
                   "value": round(T / a * 1e3), "ms_per_step": round(a, 4), f"{other}_equal_size": round(T / b * 1e3),
                   f"{other}_ms_per_step": round(b, 4), "params_b": round(new.num_params() / 1e9, 2),
                   f"{other}_params_b": round(old.num_params() / 1e9, 2), "dtype": "bf16", "data": "synthetic"}
            print(json.dumps(row), flush=True)
            out.append(row)
        del timers
        torch.cuda.empty_cache()
    return out
