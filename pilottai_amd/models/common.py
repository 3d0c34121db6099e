"""What the model families beside Llama share: packed projections, checkpoint access, looped stacks."""
from __future__ import annotations

import os
from typing import Callable, List, Optional, Tuple

import torch
import torch.nn.functional as F

from pilottai_amd import ops
from pilottai_amd.ops.latent import pad_to


class PackedLinear:
    """y = x W^T with W [N, K] padded to [128 n, 64 k] by zeros: the packed projections in bf16
    (decode kernel up to 64 rows, prefill kernel above), the library's fp32 GEMM in fp32."""

    def __init__(self, w: torch.Tensor, dtype, device):
        N, K = w.shape
        full = torch.zeros(pad_to(N, 128), pad_to(K, 64), dtype=dtype, device=device)
        full[:N, :K] = w.to(device=device, dtype=dtype)
        self.N, self.K = full.shape
        self.w = ops.pack_decode_weight(full) if dtype == torch.bfloat16 else full

    def __call__(self, x: torch.Tensor) -> torch.Tensor:
        if self.w.dim() == 2:
            return F.linear(x, self.w)
        if x.shape[0] <= 64:
            return ops.decode_gemm(x, self.w)
        return ops.prefill_gemm(x, self.w)


def pad_heads(w: torch.Tensor, padded: int) -> torch.Tensor:
    """[heads, size, k] -> [heads, padded, k], zeros behind every head."""
    out = w.new_zeros(w.shape[0], padded, w.shape[2])
    out[:, :w.shape[1]] = w
    return out


def checkpoint_reader(path: str) -> Callable:
    """get(name, shape) over a folder's *.safetensors, checking that the tensor is there and has the shape; get.shape(name)
    for a size that no configuration gives."""
    from safetensors import safe_open

    where = {}
    for f in sorted(os.listdir(path)):
        if f.endswith(".safetensors"):
            fh = safe_open(os.path.join(path, f), framework="pt")
            where.update({k: fh for k in fh.keys()})

    def file(name):
        if name not in where:
            raise ValueError(f"{path}: tensor {name!r} is missing")
        return where[name]

    def get(name, shape):
        t = file(name).get_tensor(name)
        if tuple(t.shape) != tuple(shape):
            raise ValueError(f"{path}: {name} has shape {tuple(t.shape)}, the configuration gives {tuple(shape)}")
        return t
    get.shape = lambda name: tuple(file(name).get_slice(name).get_shape())
    return get


def parse_loop(loop: Optional[dict], layers: int) -> Optional[Tuple[int, int, int]]:
    """(start, stop, times) of a config's loop entry."""
    if not loop:
        return None
    out = (int(loop["start"]), int(loop["stop"]), int(loop["times"]))
    if not (0 <= out[0] < out[1] <= layers and out[2] >= 1):
        raise ValueError(f"loop {out} does not fit {layers} layers")
    return out


def layer_runs(layers: int, loop: Optional[Tuple[int, int, int]]) -> List[Tuple[int, bool]]:
    """(layer, whether a repeated pass starts here) for every layer run of a step, in order."""
    start, stop, times = loop or (0, 0, 1)
    out = []
    for again in range(times):
        lo = start if again else 0
        out += [(i, again > 0 and i == start) for i in range(lo, stop)]
    return out + [(i, False) for i in range(stop, layers)]


def expert_tile_rows(rows: float, dtype, min_k: int, above_64: int, above_256: int) -> int:
    """Rows per sorted tile of the grouped projections: 16 streams the weights, 64 shares them, 256 runs the
    ping-pong kernels (bf16, every K of at least 128), by the rows an expert gets on average."""
    if dtype != torch.bfloat16 or rows <= above_64:
        return 16
    return 256 if min_k >= 128 and rows > above_256 else 64
