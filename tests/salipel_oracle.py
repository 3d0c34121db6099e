"""A plain, slow implementation of the Salipel design, one function per mechanism.

Everything is written out over one whole sequence: no cache, pages, batches, chunks or any code of the
product. `dt` is the arithmetic type (float64 by default, so that a comparison measures the
framework's rounding alone). Weights are stored [out, in]: W y = y @ W.T.
"""
import math

import torch

from bozupel_oracle import read_checkpoint  # noqa: F401
from mudepel_oracle import gelu_tanh, rms


def norm(x, w, eps):
    return rms(x, eps) * w


def frequencies(rot):
    """Angle per position of each pair, long waves slowed down if `scaling` is given."""
    n, base, sc = rot["dims"], rot["base"], rot.get("scaling")
    out = []
    for i in range(n // 2):
        f = base ** (-2.0 * i / n)
        if sc:
            wave = 2 * math.pi / f
            if wave > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif wave >= sc["original"] / sc["high"]:
                s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
                f = (1 - s) * f / sc["factor"] + s * f
        out.append(f)
    return torch.tensor(out, dtype=torch.float64)


def rotate(x, rot):
    """x [T, heads, n] at positions 0 .. T - 1: dimension i turns with i + dims / 2, the rest stay."""
    half = rot["dims"] // 2
    a = torch.arange(x.shape[0], dtype=torch.float64)[:, None, None] * frequencies(rot)
    c, s = a.cos().to(x.dtype), a.sin().to(x.dtype)
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], -1)


def visible(T, window=0, keep=0, chunk=0):
    """[T, T]: query i sees key j <= i; of those the last `window` and the first `keep`, or those of its chunk."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    if window:
        seen &= (i - j < window) | (j < keep)
    if chunk:
        seen &= i // chunk == j // chunk
    return seen


def attend(q, k, v, scale, seen, slope=0.0, cap=0.0, sink=None):
    """One head. q [T, n], k [T, n], v [T, m]: softmax over the seen keys and the sink's exp."""
    T = q.shape[0]
    s = q @ k.T * scale
    if cap:
        s = cap * torch.tanh(s / cap)
    s = s - slope * (torch.arange(T)[:, None] - torch.arange(T)[None, :]).to(s.dtype)
    s = s.masked_fill(~seen, -math.inf)
    top = s.max(1, keepdim=True).values
    if sink is not None:
        top = top.clamp(min=float(sink))
    e = torch.exp(s - top)
    total = e.sum(1, keepdim=True)
    if sink is not None:
        total = total + torch.exp(sink - top)
    return e / total @ v


def gate(y, h, w):
    return y * torch.sigmoid(h @ w["g"].T)


def window_attention(h, m, w, eps):
    """Rotated, normed queries and keys; the values are the keys as projected; window and kept first tokens."""
    T, H, G, n = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q, k = (h @ w["q"].T).reshape(T, H, n), (h @ w["k"].T).reshape(T, G, n)
    v = k
    q, k = rotate(norm(q, w["q.norm"], eps), m["rot"]), rotate(norm(k, w["k.norm"], eps), m["rot"])
    mask = m.get("mask") or {}
    seen = visible(T, mask.get("size", 0), mask.get("keep_first", 0))
    out = [attend(q[:, i], k[:, i // (H // G)], v[:, i // (H // G)], m["scale"], seen) for i in range(H)]
    return gate(torch.cat(out, 1), h, w) @ w["o"].T


def matrix_memory(q, k, v, i, f):
    """Token by token. q and k [T, H, N], v [T, H, V], log gates i and f [T, H] -> [T, H, V]."""
    T, H, N = q.shape
    S, n, m = q.new_zeros(H, N, v.shape[2]), q.new_zeros(H, N), q.new_zeros(H)
    out = torch.empty_like(v)
    for t in range(T):
        top = torch.maximum(f[t] + m, i[t])
        old, new = torch.exp(f[t] + m - top), torch.exp(i[t] - top)
        S = old[:, None, None] * S + new[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = old[:, None] * n + new[:, None] * k[t]
        m = top
        den = torch.maximum((n * q[t]).sum(1).abs(), torch.exp(-m)) + 1e-6
        out[t] = (S * q[t][:, :, None]).sum(1) / den[:, None]
    return out


def mlstm(h, m, w, eps):
    T, H, N, V, cap = h.shape[0], m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    q, k = (h @ w["q"].T).reshape(T, H, N) * N ** -0.5, (h @ w["k"].T).reshape(T, H, N)
    v = (h @ w["v"].T).reshape(T, H, V)
    i = cap * torch.tanh((h @ w["i"].T + w["i.b"]) / cap)
    f = torch.nn.functional.logsigmoid(cap * torch.tanh((h @ w["f"].T + w["f.b"]) / cap))
    o = rms(matrix_memory(q, k, v, i, f), eps).reshape(T, H * V) * w["norm"]
    return gate(o, h, w) @ w["o"].T


def part(w, name):
    return {k[len(name):]: v for k, v in w.items() if k.startswith(name)}


def parallel(h, m, w, eps):
    return m["left_scale"] * window_attention(h, m["left"], part(w, "left."), eps) + \
        m["right_scale"] * mlstm(h, m["right"], part(w, "right."), eps)


def chunk_attention(h, m, w, eps):
    """No rotation: a bias by distance; normed values; chunks; a sink per head."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q, k = (h @ w["q"].T).reshape(T, H, m["dim"]), (h @ w["k"].T).reshape(T, G, m["dim"])
    v = rms((h @ w["v"].T).reshape(T, G, m["vdim"]), eps)
    seen = visible(T, chunk=(m.get("mask") or {}).get("size", 0))
    out = [attend(q[:, i], k[:, i // (H // G)], v[:, i // (H // G)], m["scale"], seen, slope=2.0 ** (-8.0 * (i + 1) / H),
                  sink=w["sink"][i]) for i in range(H)]
    return torch.cat(out, 1) @ w["o"].T


def differential_lambda(w, diff):
    return torch.exp((w["lq1"] * w["lk1"]).sum()) - torch.exp((w["lq2"] * w["lk2"]).sum()) + diff


def differential(a1, a2, lam, diff, eps):
    return rms(a1 - lam * a2, eps) * (1 - diff)


def differential_attention(h, m, w, eps):
    """Two maps per head over the same values, the second one taken off the first."""
    T, H, G, n = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q, k = (h @ w["q"].T).reshape(T, H * 2, n), (h @ w["k"].T).reshape(T, G * 2, n)
    q, k = rotate(norm(q, w["q.norm"], eps), m["rot"]), rotate(norm(k, w["k.norm"], eps), m["rot"])
    v = (h @ w["v"].T).reshape(T, G, m["vdim"])
    lam, seen, out = differential_lambda(w, m["diff"]), visible(T), []
    for i in range(H):
        g = i // (H // G)
        a = [attend(q[:, 2 * i + c], k[:, 2 * g + c], v[:, g], m["scale"], seen, cap=m["softcap"]) for c in (0, 1)]
        out.append(differential(a[0], a[1], lam, m["diff"], eps))
    return gate(torch.cat(out, 1), h, w) @ w["o"].T


def route(h, w_router, correction, r):
    """[T, experts] weights, zero where an expert is not chosen."""
    s = torch.softmax(h @ w_router.T, -1)
    top = (s + correction).topk(r["top"], -1).indices
    kept = torch.zeros_like(s).scatter_(1, top, s.gather(1, top))
    return kept / (kept.sum(1, keepdim=True) + 1e-20) * r["scale"]


def feed_forward(h, p, w):
    if p["kind"] == "dense":
        return (gelu_tanh(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T
    wt = route(h, w["router"], w["correction"], p["router"])
    return sum(wt[:, e:e + 1] * (torch.relu(h @ w[f"e{e}.up"].T) ** 2 @ w[f"e{e}.down"].T) for e in range(wt.shape[1]))


MIXERS = {"parallel": parallel, "attention": chunk_attention, "attention_2": differential_attention}


def forward(cfg, tensors, ids, dt=torch.float64, layers=None):
    """Logits [T, vocab] of one sequence; `layers` (a list) collects the residual after every layer."""
    tw = {k: (v.to(dt) if v.is_floating_point() else v) for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    x = tw["embed"][torch.tensor(list(ids))]
    for i, L in enumerate(cfg["layers"]):
        w = part(tw, f"l{i}.")
        h = norm(x, w["norm1"], eps)
        y = MIXERS[L["type"]](h, L["mixer"], part(w, "mix."), eps)
        if L.get("mlp"):
            y = y + feed_forward(h, L["mlp"], part(w, "mlp."))
        x = x + cfg["residual_mult"] * y
        if layers is not None:
            layers.append(x)
    return norm(x, tw["final.norm"], eps) @ tw["head"].T
