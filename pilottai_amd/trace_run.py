"""Trace replay: feed given token ids through a served model, step by step, and write logits.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Steps come from standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

All entries of a step run as one batch (LLMEngine.feed_step: the scheduler, paged cache and forward
that generation uses). The logits at the wanted places go to OUT/<step>.f32 as little-endian fp32
[wanted, vocab], in order; then "done <step>" is printed. Requests named in "end" give back their
pages and state slots. The cache pool holds N tokens and four requests may be live, so pages and slots are used
again. Kernels that are not built yet are compiled first, only those the model needs.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

SLOTS = 4  # live requests
PAGE_TOKENS = 64  # a request's share of the pool is counted in these


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(description="Replay a trace of token ids and write the logits it asks for.")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="tokens the live requests hold at most, each rounded up to 64: the size of the cache pool")
    ap.add_argument("--device", default=None, help="cuda (default) or cpu: the fp32 reference operations, slow")
    a = ap.parse_args(argv)
    if a.max_tokens < 1:
        ap.error("--max-tokens must be positive")

    from pilottai_amd import _build

    from pilottai_amd.models import registry

    _build.ensure(registry.model_class(registry.get_config(a.model)).KERNELS, gpu=a.device != "cpu")
    import torch

    from pilottai_amd.engine.engine import EngineConfig, LLMEngine

    if a.device != "cpu" and not torch.cuda.is_available():
        print("trace_run: no GPU (use --device cpu for the reference operations)", file=sys.stderr)
        return 2
    torch.backends.cuda.matmul.allow_tf32 = False
    n = (a.max_tokens + PAGE_TOKENS - 1) // PAGE_TOKENS * PAGE_TOKENS
    eng = LLMEngine(EngineConfig(model=a.model, dtype=a.dtype, max_num_seqs=SLOTS, max_num_batched_tokens=n,
                                 max_model_len=n, num_kv_blocks=n // 16, exact_kv_blocks=True, prefix_caching=False,
                                 use_graphs=False),
                    device=torch.device(a.device or "cuda:0"))
    os.makedirs(a.out, exist_ok=True)
    ids = {}
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        entries = [(ids.setdefault(e["id"], eng.new_request_id()), e["tokens"], e.get("want", ()))
                   for e in step["entries"]]
        if entries:
            logits = eng.feed_step(entries)
            if logits.shape[0]:
                logits.cpu().numpy().astype("<f4").tofile(os.path.join(a.out, f"{step['step']}.f32"))
        for name in step.get("end", ()):
            eng.release_fed(ids.pop(name))
        print(f"done {step['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
