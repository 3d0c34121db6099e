"""A plain, slow implementation of the Pusunex design, one function per mechanism.

Everything is written out over one whole sequence: no cache, pages, batches, chunks, absorbed products or any code of
the product. `dt` is the arithmetic type (float64 by default, so that a comparison measures the framework's rounding
alone). Weights are stored [out, in]: W y = y @ W.T.
"""
import math

import torch

from bozupel_oracle import read_checkpoint  # noqa: F401
from mudepel_oracle import gelu_tanh, rms, silu
from salipel_oracle import part


def rms_norm(x, w, eps):
    return rms(x, eps) * w


def group_norm(x, w, eps, groups):
    """Each of `groups` equal parts of the vector by its own root mean square, then the whole times w."""
    return rms(x.reshape(*x.shape[:-1], groups, -1), eps).reshape(x.shape) * w


def rotate_pairs(x, rot):
    """x [T, heads, n] at positions 0 .. T - 1: dimension 2 i turns with dimension 2 i + 1 by position * base^(-2 i / dims)."""
    out = x.clone()
    pos = torch.arange(x.shape[0], dtype=torch.float64)[:, None]
    for i in range(rot["dims"] // 2):
        a = pos * rot["base"] ** (-2.0 * i / rot["dims"])
        c, s = a.cos().to(x.dtype), a.sin().to(x.dtype)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i], out[..., 2 * i + 1] = u * c - v * s, v * c + u * s
    return out


def causal_softmax(scores):
    """[T, T] scores of queries (rows) and keys -> weights over the keys at and before each query."""
    T = scores.shape[0]
    return torch.softmax(scores.masked_fill(torch.arange(T)[:, None] < torch.arange(T)[None, :], -math.inf), 1)


def latent(h, w, rank, eps):
    """What a layer caches of a token: the normed latent, and the rest of the same projection as it is."""
    a = h @ w["dkv"].T
    return rms_norm(a[:, :rank], w["dkv.norm"], eps), a[:, rank:]


def latent_heads(c, m, w):
    """Keys and values of every head, [T, H, dim] and [T, H, vdim], from the latents."""
    T, H = c.shape[0], m["heads"]
    return (c @ w["uk"].T).reshape(T, H, m["dim"]), (c @ w["uv"].T).reshape(T, H, m["vdim"])


def attend_latent(h, c, m, w):
    """No positions; `c`: this layer's latents, or another one's; output gate."""
    T, H = h.shape[0], m["heads"]
    q = (h @ w["q"].T).reshape(T, H, m["dim"])
    k, v = latent_heads(c, m, w)
    o = torch.cat([causal_softmax(q[:, i] @ k[:, i].T * m["scale"]) @ v[:, i] for i in range(H)], 1)
    return (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def attend_latent_rotated(h, m, w, eps):
    """Queries through a latent of their own; a rotated part beside the unrotated one, whose key all heads share."""
    T, H, n, r = h.shape[0], m["heads"], m["dim"], m["rot_dim"]
    q = (rms_norm(h @ w["dq"].T, w["dq.norm"], eps) @ w["uq"].T).reshape(T, H, n + r)
    c, kr = latent(h, w, m["kv_rank"], eps)
    k, v = latent_heads(c, m, w)
    qr, kr = rotate_pairs(q[..., n:], m["rot"]), rotate_pairs(kr[:, None], m["rot"])[:, 0]
    o = [causal_softmax((q[:, i, :n] @ k[:, i].T + qr[:, i] @ kr.T) * m["scale"]) @ v[:, i] for i in range(H)]
    return torch.cat(o, 1) @ w["o"].T, c


def log_decay(h, w, tau):
    """log of sigmoid(z)^(1 / tau) per key channel, [T, heads * dim]."""
    return torch.nn.functional.logsigmoid((h @ w["a1"].T) @ w["a2"].T + w["a2.b"]) / tau


def linear_memory(q, k, v, g, S=None):
    """Token by token. q, k and log decays g [T, H, N], v [T, H, V] -> o [T, H, V] and the state [H, N, V]."""
    T, H, N = q.shape
    S = q.new_zeros(H, N, v.shape[2]) if S is None else S
    o = torch.empty_like(v)
    for t in range(T):
        S = torch.exp(g[t])[:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    return o, S


def gated_linear_attention(h, m, w, eps):
    T, H, N, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k = (h @ w["q"].T).reshape(T, H, N) * N ** -0.5, (h @ w["k"].T).reshape(T, H, N)
    o, _ = linear_memory(q, k, (h @ w["v"].T).reshape(T, H, V), log_decay(h, w, m["tau"]).reshape(T, H, N))
    return (rms_norm(o, w["norm"], eps).reshape(T, H * V) * silu(h @ w["g"].T)) @ w["o"].T


def poly_norm(z, act, eps):
    a, b, c, e = act
    return a * rms(z, eps) + b * rms(z ** 2, eps) + c * rms(z ** 3, eps) + e


def expert(h, w):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def route(h, w_router, top):
    """[T, experts] weights, zero where an expert is not chosen."""
    s = torch.sigmoid(h @ w_router.T)
    at = s.topk(top, -1).indices
    return torch.zeros_like(s).scatter_(1, at, s.gather(1, at))


def feed_forward(h, p, w, eps):
    if p["kind"] == "dense":
        return poly_norm(h @ w["up"].T, w["act"], eps) @ w["down"].T
    wt = route(h, w["router"], p["router"]["top"])
    y = expert(h, part(w, "shared.")) if p.get("shared") else torch.zeros_like(h)
    for e in range(wt.shape[1]):
        used = wt[:, e] > 0
        if used.any():
            y[used] += expert(wt[used, e:e + 1] * h[used], part(w, f"e{e}."))
    return y


def token_side(x, e, w, eps):
    return rms_norm((gelu_tanh(x @ w["gate"].T) * e) @ w["proj"].T, w["norm"], eps)


def depth_average(xs, a):
    return sum(a[j] * xs[j] for j in range(len(xs)))


def forward(cfg, tensors, ids, dt=torch.float64, layers=None):
    """Logits [T, vocab] of one sequence; `layers` (a list) collects what goes on behind every layer."""
    tw = {k: (v.to(dt) if v.is_floating_point() else v) for k, v in tensors.items()}
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    ids = torch.tensor(list(ids))
    x = tw["embed"][ids]
    xs, latents = [x], {}
    for i, L in enumerate(cfg["layers"]):
        w, m = part(tw, f"l{i}."), L["mixer"]
        mix = part(w, "mix.")
        h = group_norm(x, w["norm1"], eps, groups)
        if L["type"] == "gla":
            y = gated_linear_attention(h, m, mix, eps)
        elif L["type"] == "latent_attention_2":
            y, latents[i] = attend_latent_rotated(h, m, mix, eps)
        else:
            if m.get("kv_from") is None:
                latents[i], _ = latent(h, mix, m["kv_rank"], eps)
            y = attend_latent(h, latents[i if m.get("kv_from") is None else m["kv_from"]], m, mix)
        x = x + group_norm(y, w["norm1b"], eps, groups)
        if L.get("mlp"):
            h = group_norm(x, w["norm2"], eps, groups)
            x = x + group_norm(feed_forward(h, L["mlp"], part(w, "mlp."), eps), w["norm2b"], eps, groups)
        dim = cfg["token_side"]["dim"]
        x = x + token_side(x, tw["side.embed"][ids][:, i * dim:(i + 1) * dim], part(w, "side."), eps)
        xs.append(x)
        x = depth_average(xs, w["dwa"])
        if layers is not None:
            layers.append(x)
    return group_norm(x, tw["final.norm"], eps, groups) @ tw["head"].T
