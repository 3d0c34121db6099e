"""A plain, slow implementation of the Mudepel design, one function per mechanism.

Everything is written out over one whole sequence: no cache, pages, batches, chunks or any code of the
product. `dt` is the arithmetic type (float64 by default, so that a comparison measures the
framework's rounding alone). Weights are stored [out, in]: W y = y @ W.T.
"""
import math

import torch

from bozupel_oracle import read_checkpoint  # noqa: F401


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, w, eps):
    return rms(x, eps) * (1 + w)


def silu(x):
    return x * torch.sigmoid(x)


def gelu_tanh(x):
    return 0.5 * x * (1 + torch.tanh(math.sqrt(2 / math.pi) * (x + 0.044715 * x ** 3)))


def frequencies(rot):
    """(angle per position for each pair, factor of cos and sin)."""
    n, base, sc = rot["dims"], rot["base"], rot.get("scaling")
    f = [base ** (-2.0 * i / n) for i in range(n // 2)]
    if not sc:
        return torch.tensor(f, dtype=torch.float64), 1.0
    where = lambda turns: n * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))  # noqa: E731
    lo, hi = max(math.floor(where(sc["fast"])), 0), min(math.ceil(where(sc["slow"])), n - 1)
    out = []
    for i, x in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(x / sc["factor"] * r + x * (1 - r))
    return torch.tensor(out, dtype=torch.float64), 0.1 * math.log(sc["factor"]) + 1


def rotate(x, rot):
    """x [T, heads, n] at positions 0 .. T - 1."""
    half = rot["dims"] // 2
    f, m = frequencies(rot)
    a = torch.arange(x.shape[0], dtype=torch.float64)[:, None, None] * f
    c, s = (a.cos() * m).to(x.dtype), (a.sin() * m).to(x.dtype)
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], -1)


def pooled_attention(q, k, v, scale, window, pool, sink=1.0):
    """One head. q [T, n], k [T, n], v [T, m]: query i sees keys j with 0 <= i - j < window and the mean of
    every whole block of `pool` keys that ends at or before i - window; exp(s) / (sink + sum exp(s))."""
    T = q.shape[0]
    back = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    seen = (back >= 0) & (back < window) if window else back >= 0
    keys, vals = k, v
    if pool and window and T // pool:
        n = T // pool
        keys = torch.cat([k, k[:n * pool].reshape(n, pool, -1).mean(1)])
        vals = torch.cat([v, v[:n * pool].reshape(n, pool, -1).mean(1)])
        last = torch.arange(n) * pool + pool - 1
        seen = torch.cat([seen, last[None, :] <= torch.arange(T)[:, None] - window], 1)
    s = (q @ keys.T * scale).masked_fill(~seen, -math.inf)
    top = s.max(1, keepdim=True).values
    if sink:
        top = top.clamp(min=0)
    e = torch.exp(s - top)
    return e / ((sink * torch.exp(-top) if sink else 0) + e.sum(1, keepdim=True)) @ vals


def attention(h, m, w):
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    lin = lambda x, n: x @ w[n].T + w[n + ".b"]  # noqa: E731
    q = rotate(lin(h, "q").reshape(T, H, m["dim"]), m["rot"])
    k = rotate(lin(h, "k").reshape(T, G, m["dim"]), m["rot"])
    v = lin(h, "v").reshape(T, G, m["vdim"])
    mask = m.get("mask") or {}
    out = [pooled_attention(q[:, i], k[:, i // (H // G)], v[:, i // (H // G)], m["scale"], mask.get("size"), mask.get("pool"))
           for i in range(H)]
    return lin(torch.cat(out, 1), "o")


def causal_conv(x, w, b):
    """x [T, channels], w [channels, taps], the last tap at the current token."""
    T, taps = x.shape[0], w.shape[1]
    pad = torch.cat([x.new_zeros(taps - 1, x.shape[1]), x])
    return b + sum(pad[k:k + T] * w[:, k] for k in range(taps))


def state_scan(x, B, C, dt, A, D):
    """Token by token. x [T, H, V], B and C [T, H, N], dt [T, H], A and D [H]."""
    T, H, V = x.shape
    S, out = x.new_zeros(H, B.shape[2], V), torch.empty_like(x)
    for t in range(T):
        S = torch.exp(A * dt[t])[:, None, None] * S + dt[t][:, None, None] * B[t][:, :, None] * x[t][:, None, :]
        out[t] = (S * C[t][:, :, None]).sum(1) + D[:, None] * x[t]
    return out


def mamba2(h, m, w, eps):
    T, H, V, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * V
    z, xbc, dt = torch.split(h @ w["in"].T, [inner, inner + 2 * G * N, H], 1)
    x, B, C = torch.split(silu(causal_conv(xbc, w["conv"], w["conv.b"])), [inner, G * N, G * N], 1)
    dt = torch.nn.functional.softplus(dt + w["dt_bias"], threshold=1e9)
    share = lambda y: y.reshape(T, G, N).repeat_interleave(H // G, 1)  # noqa: E731
    y = state_scan(x.reshape(T, H, V), share(B), share(C), dt, -torch.exp(w["A_log"]), w["D"]).reshape(T, inner)
    parts = (y * silu(z)).reshape(T, m["norm_groups"], -1)
    return (rms(parts, eps).reshape(T, inner) * w["norm"]) @ w["o"].T


def gated(h, w, pre, act):
    return (act(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def route(h, w_router, r):
    """[T, experts] weights, zero where an expert is not chosen."""
    s = torch.sigmoid(h @ w_router.T)
    T, E = s.shape
    g = r.get("groups") or {"count": 1, "keep": 1}
    per = s.reshape(T, g["count"], E // g["count"])
    best = per.topk(min(2, per.shape[2]), -1).values.sum(-1).topk(g["keep"], -1).indices
    ok = torch.zeros(T, g["count"], dtype=torch.bool).scatter_(1, best, True).repeat_interleave(E // g["count"], 1)
    top = s.masked_fill(~ok, -1).topk(r["top"], -1).indices
    return torch.zeros_like(s).scatter_(1, top, s.gather(1, top))


def experts(h, p, w):
    wt = route(h, w["router"], p["router"])
    y = sum(wt[:, e:e + 1] * gated(h, w, f"e{e}.", silu) for e in range(wt.shape[1]))
    return y + gated(h, w, "shared.", silu) if p.get("shared") else y


def feed_forward(h, p, w):
    return gated(h, w, "", gelu_tanh) if p["kind"] == "dense" else experts(h, p, w)


def runs(cfg):
    """The layers in the order they run."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return list(range(n))
    a, b = lp["start"], lp["stop"]
    return list(range(a)) + list(range(a, b)) * lp["times"] + list(range(b, n))


def hyper(X, w, q, sub):
    """X [streams, T, D]: one sublayer of a hyper-connected residual."""
    y = sub((w[f"hc{q}.in"][:, None, None] * X).sum(0))
    mixed = torch.stack([(w[f"hc{q}.mix"][:, t][:, None, None] * X).sum(0) for t in range(X.shape[0])])
    return mixed + w[f"hc{q}.out"][:, None, None] * y


def forward(cfg, tensors, ids, dt=torch.float64, layers=None):
    """Logits [T, vocab] of one sequence; `layers` (a list) collects the sum of the streams after every layer run."""
    tw = {k: (v.to(dt) if v.is_floating_point() else v) for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    X = tw["embed"][torch.tensor(list(ids))].expand(cfg["streams"], -1, -1)
    for i in runs(cfg):
        L, w = cfg["layers"][i], {k[len(f"l{i}."):]: v for k, v in tw.items() if k.startswith(f"l{i}.")}
        sub = lambda pre: {k[len(pre):]: v for k, v in w.items() if k.startswith(pre)}  # noqa: E731
        mix = (lambda h: attention(h, L["mixer"], sub("mix."))) if L["type"] == "attention" else \
            (lambda h: mamba2(h, L["mixer"], sub("mix."), eps))
        X = hyper(X, w, 1, lambda u: mix(norm(u, w["norm1"], eps)))
        if L["mlp"] is not None:
            X = hyper(X, w, 2, lambda u: feed_forward(norm(u, w["norm2"], eps), L["mlp"], sub("mlp.")))
        if layers is not None:
            layers.append(X.sum(0))
    z = norm(X.sum(0), tw["final.norm"], eps) @ tw["embed"].T
    cap = cfg.get("logit_softcap")
    return cap * torch.tanh(z / cap) if cap else z
