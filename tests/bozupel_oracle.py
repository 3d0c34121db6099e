"""A plain, slow implementation of the Bozupel design, one function per mechanism.

Everything is written out over one whole sequence, without a cache, pages, batches or any code
of the product. The tests compare the framework with it. `dt` is the arithmetic type (float64 by
default, so that the comparison measures the framework's rounding alone).

Notation: x residual [T, D], h a sublayer's input, W y = y @ W.T (weights are stored [out, in]).
"""
import json
import math
import os
import struct

import numpy as np
import torch


def read_checkpoint(path):
    """name -> tensor of a folder's model.safetensors (header length, JSON header, raw data)."""
    raw = open(os.path.join(path, "model.safetensors"), "rb").read()
    n = struct.unpack("<Q", raw[:8])[0]
    head, body = json.loads(raw[8:8 + n]), raw[8 + n:]
    out = {}
    for name, m in head.items():
        if name == "__metadata__":
            continue
        a, b = m["data_offsets"]
        if m["dtype"] == "BF16":
            bits = np.frombuffer(body[a:b], dtype="<u2").astype(np.uint32) << 16
            t = torch.from_numpy(bits.view(np.float32).copy())
        else:
            t = torch.from_numpy(np.frombuffer(body[a:b], dtype={"I32": "<i4", "F32": "<f4"}[m["dtype"]]).copy())
        out[name] = t.reshape(m["shape"])
    return out


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def rotate(x, pos, dims, base):
    """x [T, ..., n]: dimension i < dims/2 turns with dimension i + dims/2 by pos * base^(-2i/dims)."""
    half = dims // 2
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=torch.float64)
    a = (pos.double()[:, None] * f[None, :]).reshape(len(pos), *([1] * (x.dim() - 2)), half)
    c, s = a.cos().to(x.dtype), a.sin().to(x.dtype)
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], -1)


def visible(T, window):
    """[T, T] bool: query i sees key j with 0 <= i - j < window (no window: every j <= i)."""
    d = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    return (d >= 0) & (d < window) if window else d >= 0


def latent_attention(h, m, w, eps):
    """w: the mixer's tensors by their short names (dq, dq.norm, uq, dkv, dkv.norm, uk, uv, o)."""
    T, H = h.shape[0], m["heads"]
    n, r, vd, R = m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(T)
    rd, base = m["rot"].get("dims", r), m["rot"]["base"]
    q = (rms_norm(h @ w["dq"].T, w["dq.norm"], eps) @ w["uq"].T).reshape(T, H, n + r)
    q_rot = rotate(q[..., n:], pos, rd, base)
    kv = h @ w["dkv"].T
    c = rms_norm(kv[:, :R], w["dkv.norm"], eps)
    k_rot = rotate(kv[:, R:], pos, rd, base)
    k = (c @ w["uk"].T).reshape(T, H, n)
    v = (c @ w["uv"].T).reshape(T, H, vd)
    mask = visible(T, (m.get("mask") or {}).get("size"))
    out = torch.empty(T, H, vd, dtype=h.dtype)
    for i in range(H):
        s = (q[:, i, :n] @ k[:, i].T + q_rot[:, i] @ k_rot.T) * m["scale"]
        s = s.masked_fill(~mask, -math.inf)
        out[:, i] = torch.softmax(s, -1) @ v[:, i]
    return out.reshape(T, H * vd) @ w["o"].T


def expert(h, w_gate, w_up, w_down, limit):
    g = (h @ w_gate.T).clamp(max=limit)
    u = (h @ w_up.T).clamp(-limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ w_down.T


def table_experts(h, ids, p, w):
    """p: the config's 'mlp' entry; token t goes through the experts of row ids[t] of the table."""
    top = p["router"]["top"]
    y = torch.zeros_like(h)
    for t, token in enumerate(ids):
        for e in w["table"][token].tolist():
            y[t] += expert(h[t:t + 1], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], p["expert"]["limit"])[0] / top
    return y


def passes(cfg):
    """The layer indices in the order they run, and for each whether a repeated pass starts there."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    a, b = lp["start"], lp["stop"]
    run = [(i, False) for i in range(b)]
    for _ in range(lp["times"] - 1):
        run += [(i, i == a) for i in range(a, b)]
    return run + [(i, False) for i in range(b, n)]


def forward(cfg, tensors, ids, dt=torch.float64, layers=None):
    """Logits [T, vocab] of one sequence; `layers` (a list) collects the residual after every layer run."""
    tw = {k: (v.to(dt) if v.is_floating_point() else v) for k, v in tensors.items()}

    def sub(prefix):
        return {k[len(prefix):]: v for k, v in tw.items() if k.startswith(prefix)}

    eps = cfg["norm"]["eps"]
    ids = list(ids)
    first = tw["embed"][torch.tensor(ids)]
    x = first
    for i, again in passes(cfg):
        if again:
            x = x + first
        L, p = cfg["layers"][i], f"l{i}."
        y = latent_attention(rms_norm(x, tw[p + "norm1"], eps), L["mixer"], sub(p + "mix."), eps)
        x = x + rms_norm(y, tw[p + "norm1b"], eps)
        if L["mlp"] is not None:
            y = table_experts(rms_norm(x, tw[p + "norm2"], eps), ids, L["mlp"], sub(p + "mlp."))
            x = x + rms_norm(y, tw[p + "norm2b"], eps)
        if layers is not None:
            layers.append(x)
    return rms_norm(x, tw["final.norm"], eps) @ tw["head"].T * cfg["logit_scale"]
