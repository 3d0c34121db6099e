"""The operations that the Pusunex design brings, each alone (reference operations on the CPU; kernels on the GPU in
bf16 and fp32) against the plain functions of tests/pusunex_oracle.py, at sizes that are not whole tiles."""
import math

import numpy as np
import pytest
import torch

import pusunex_oracle as oracle
from test_hybrid_kernels import BF16, F32, fed_step, gen, kinds, tol


# ---- residual ----------------------------------------------------------------------------------------
ROWS = [(72, 3, 2), (256, 2, 2), (50, 1, 5), (160, 5, 1), (640, 5, 10), (1536, 3, 1), (2048, 4, 8), (4096, 8, 2), (8192, 1, 16),
        (96, 6, 4), (2056, 1, 1), (12288, 2, 1)]


@kinds
@pytest.mark.parametrize("T", [9, 1030])
@pytest.mark.parametrize("D,post,nxt", ROWS)
def test_group_norms(device, dt, D, post, nxt, T):
    """x + n(sum of partial outputs), the next norm; and the sum itself as the next projection's input."""
    from pilottai_amd import ops

    if T > 9 and (device == "cpu" or D > 4096 and dt == F32):
        T = 17
    g, K, ld, eps = gen(D + T), 3, (D + 63) // 64 * 64, 1e-3
    r, y = torch.randn(T, D, generator=g), torch.randn(T * K, ld, generator=g).to(dt)
    y[:, :D // post] *= 30  # (parts of unlike size)
    wp, wn = torch.rand(D, generator=g) + 0.5, torch.rand(D, generator=g) + 0.5
    want = r.double() + oracle.group_norm(y.double()[:, :D].view(T, K, D).sum(1), wp.double(), eps, post)
    d = lambda t: t.to(device)  # noqa: E731
    for w in (wn, None):
        rg, out = d(r).clone(), torch.full((T, ld), 7.0, dtype=dt, device=device)
        ops.residual_norm(rg, eps, y=d(y), partials=K, w_post=d(wp), post_groups=post, w_next=None if w is None else d(w),
                          next_groups=nxt if w is not None else 1, out=out)
        torch.testing.assert_close(rg.double().cpu(), want, rtol=1e-5, atol=1e-4)
        torch.testing.assert_close(out.double().cpu()[:, :D], want if w is None else oracle.group_norm(want, wn.double(), eps, nxt), **tol(dt))
        assert not out[:, D:].any()


@kinds
@pytest.mark.parametrize("n", [1, 2, 5])
@pytest.mark.parametrize("D,groups", [(72, 3), (256, 1), (2048, 4), (100, 4), (4096, 16)])
def test_depth_average(device, dt, D, groups, n):
    """The n-th layer's result joins the earlier ones, and their weighted sum goes on."""
    from pilottai_amd import ops

    g, T, V, ld, eps = gen(D + n), 11, 23, (D + 63) // 64 * 64, 1e-4
    r, y, w, wn = (torch.randn(T, D, generator=g), torch.randn(T, ld, generator=g).to(dt), torch.rand(D, generator=g) + 0.5,
                   torch.rand(D, generator=g) + 0.5)
    emb, ids, a = torch.randn(V, D, generator=g).to(dt), torch.randint(0, V, (T,), generator=g, dtype=torch.int32), torch.randn(n + 1, generator=g)
    hist = torch.randn(n + 1, T, D, generator=g)
    x = r.double() + oracle.rms_norm(y.double()[:, :D], w.double(), eps)
    want = oracle.depth_average([emb[ids.long()].double(), *hist[:n - 1].double(), x], a.double())
    h = oracle.group_norm(want, wn.double(), eps, groups)
    d = lambda t: t.to(device)  # noqa: E731
    kw = dict(y=d(y), w_post=d(w), emb=d(emb), ids=d(ids), mix=d(a), w_next=d(wn), next_groups=groups)
    rows = torch.tensor([10, 3, 3, 0], dtype=torch.int32)
    rg, hg, out = d(r).clone(), d(hist).clone(), torch.full((4, ld), 7.0, dtype=dt, device=device)
    ops.residual_norm(rg, eps, out=out, hist=hg, rows=d(rows), **kw)  # leaves everything alone
    assert torch.equal(rg.cpu(), r) and torch.equal(hg.cpu(), hist)
    torch.testing.assert_close(out.double().cpu()[:, :D], h[rows.long()], **tol(dt))
    out = torch.full((T, ld), 7.0, dtype=dt, device=device)
    ops.residual_norm(rg, eps, out=out, hist=hg, **kw)
    torch.testing.assert_close(rg.double().cpu(), want, rtol=1e-5, atol=1e-4)
    torch.testing.assert_close(hg[n - 1].double().cpu(), x, rtol=1e-5, atol=1e-4)
    hg[n - 1] = d(hist[n - 1])
    assert torch.equal(hg.cpu(), hist)  # nothing else
    torch.testing.assert_close(out.double().cpu()[:, :D], h, **tol(dt))


# ---- projections with a second factor ------------------------------------------------------------------
@kinds
@pytest.mark.parametrize("T", [1, 40, 130, 700])
@pytest.mark.parametrize("G,N,K", [(3, 48, 32), (5, 208, 96), (2, 512, 128), (16, 128, 64)])
def test_gated_heads(device, dt, T, G, N, K):
    from pilottai_amd import ops

    g = gen(T + N)
    x, w = torch.randn(T, G * (K + 32), generator=g).to(dt), (torch.randn(G, N, K, generator=g) / math.sqrt(K)).to(dt)
    z = (torch.randn(T, G * (N + 16) + 24, generator=g) * 3).to(dt)
    out = torch.full((T, G * (N + 16)), 5.0, dtype=dt, device=device)
    ops.head_gemm(x.to(device), K + 32, ops.pack_groups(w, dt).to(device), out, N + 16, gate=z.to(device)[:, 8:])
    o = out.double().cpu().view(T, G, N + 16)
    want = torch.einsum("tgk,gnk->tgn", x.double().view(T, G, K + 32)[:, :, :K], w.double())
    want = want * torch.sigmoid(z.double()[:, 8:8 + G * (N + 16)].view(T, G, N + 16)[:, :, :N])
    torch.testing.assert_close(o[:, :, :N], want, **tol(dt))
    assert (o[:, :, N:] == 5.0).all()


@kinds
@pytest.mark.parametrize("T", [1, 17, 260, 3100])
@pytest.mark.parametrize("dim,d,layers", [(24, 72, 3), (256, 2048, 2), (100, 320, 1), (64, 1000, 4)])
def test_token_side(device, dt, T, dim, d, layers):
    """The token's own columns of a table, gated by the residual, and their norm."""
    from pilottai_amd.models.pusunex import TokenSide
    from pilottai_amd.ops.latent import pad_to

    if T > 300 and (device == "cpu" or dt == F32):
        T = 65
    g, V, eps, dev, dp = gen(T + d), 19, 1e-3, torch.device(device), pad_to(dim, 64)
    t = {"gate": (torch.randn(dim, d, generator=g) * 1.5 / d ** 0.5).to(BF16), "proj": (torch.randn(d, dim, generator=g) / dim ** 0.5).to(BF16),
         "norm": torch.rand(d, generator=g) + 0.5}
    tab, ids = torch.randn(V, layers, dim, generator=g).to(BF16), torch.randint(0, V, (T,), generator=g, dtype=torch.int32)
    full = torch.zeros(V, layers, dp)
    full[:, :, :dim] = tab.float()
    x = torch.zeros(T, pad_to(d, 64)).to(dt)
    x[:, :d] = torch.randn(T, d, generator=g).to(dt)
    for i in range(layers):
        mod = TokenSide(t, i * dp, d, dt, dev)
        y = mod(x.to(dev), full.view(V, -1).to(dt).to(dev), ids.to(dev)).double().cpu()[:, :d]
        w = {k: v.double() for k, v in t.items()}
        want = oracle.token_side(x.double()[:, :d], tab[ids.long(), i].double(), w, eps)
        torch.testing.assert_close(oracle.rms_norm(y, w["norm"], eps), want, **tol(dt, 3.0))


# ---- feed-forwards -------------------------------------------------------------------------------------
@kinds
@pytest.mark.parametrize("n", [33, 64, 200, 4096, 6000, 8192, 16384, 20000])
def test_poly_norm(device, dt, n):
    from pilottai_amd import ops

    g, T, eps = gen(n), 6, 1e-3
    z = torch.full((T, (n + 63) // 64 * 64 + 64), 3.0).to(dt)
    z[:, :n] = (torch.randn(T, n, generator=g) * torch.tensor([0.01, 0.3, 1.0, 2.0, 8.0, 30.0])[:, None]).to(dt)
    act = torch.tensor([0.7, -0.4, 0.9, 0.2])
    zg = z.to(device).clone()
    view = zg[:, :(n + 63) // 64 * 64]
    ops.poly_norm(view, n, act.to(device), eps)
    want = oracle.poly_norm(z[:, :n].double(), act.double(), eps)
    torch.testing.assert_close(view.double().cpu()[:, :n], want, **tol(dt, 2.0))
    assert not view[:, n:].any() and (zg[:, view.shape[1]:] == 3.0).all()


@kinds
@pytest.mark.parametrize("T", [1, 33, 150])
@pytest.mark.parametrize("d,ff", [(72, 100), (128, 256), (50, 33)])
def test_poly_feed_forward(device, dt, T, d, ff):
    from pilottai_amd.models.hybrid import PolyMLP, PolySpec
    from pilottai_amd.ops import pad_to

    g, eps = gen(T + ff), 1e-4
    t = {k: (torch.randn(s, generator=g) / s[-1] ** 0.5).to(BF16) for k, s in PolySpec(ff).shapes(d).items()}
    t["act"] = torch.tensor([0.8, 0.5, -0.6, 0.3]).to(BF16)
    h = torch.zeros(T, pad_to(d, 64)).to(dt)
    h[:, :d] = torch.randn(T, d, generator=g).to(dt)
    y = PolyMLP(PolySpec(ff), t, eps, dt, torch.device(device))(h.to(device), None)[0]
    want = oracle.feed_forward(h[:, :d].double(), {"kind": "dense"}, {k: v.double() for k, v in t.items()}, eps)
    torch.testing.assert_close(y.double().cpu()[:, :d], want, **tol(dt, 3.0))


@kinds
@pytest.mark.parametrize("T", [1, 16, 90, 700, 1500])
@pytest.mark.parametrize("E,top,ff,d,shared", [(6, 2, 40, 72, 50), (4, 1, 128, 256, 128), (9, 3, 200, 128, 0), (3, 3, 64, 192, 200)])
def test_experts_with_weighted_inputs(device, dt, T, E, top, ff, d, shared):
    """The weight is inside: an expert of w h differs from w times the expert of h. Tiles of 16, 64 and 256 rows."""
    from pilottai_amd.models.cache import StepMeta
    from pilottai_amd.models.hybrid import ScoredExperts, ScoredExpertsSpec
    from pilottai_amd.ops import pad_to

    if T == 1500 and (device == "cpu" or dt == F32):
        T = 20
    g = gen(T + d)
    spec = ScoredExpertsSpec(experts=E, top=top, ff=ff, shared_ff=shared, weigh_input=True)
    t = {k: (torch.randn(s, generator=g) / s[-1] ** 0.5 * 1.7).to(BF16) for k, s in spec.shapes(d).items()}
    mod = ScoredExperts(spec, t, d, dt, torch.device(device))
    h = torch.zeros(T, pad_to(d, 64)).to(dt)
    h[:, :d] = torch.randn(T, d, generator=g).to(dt)
    meta = StepMeta(*([None] * 2), torch.arange(T, dtype=torch.int32, device=device), *([None] * 8))
    y, K, w, _ = mod(h.to(device), meta)
    assert w is None
    got = y.double().cpu().view(T, K, -1)[:, :, :d].sum(1)
    p = {"kind": "moe", "router": {"top": top}, "shared": shared}
    tw = {k: v.double() for k, v in t.items()}
    want = oracle.feed_forward(h[:, :d].double(), p, tw, 0.0)
    ok = (got - want).abs().amax(1) < (0.06 if dt == BF16 else 2e-4) * float(want.abs().max())
    assert ok.float().mean() > 0.96  # (a close call swaps an expert)


# ---- latent attention ----------------------------------------------------------------------------------
STEPS = {"prompt": [(0, 75)], "decode": [(0, 1), (15, 1), (16, 1), (700, 1), (33, 1)], "two": [(130, 2), (0, 2)],
         "mixed": [(500, 60), (37, 1), (0, 9), (64, 1), (300, 2)], "long": [(1500, 130)]}


@kinds
@pytest.mark.parametrize("step", list(STEPS))
@pytest.mark.parametrize("H,R", [(3, 40), (8, 128), (16, 96), (20, 256), (1, 512), (5, 30), (4, 384)])
def test_latents_without_positions(device, dt, H, R, step):
    """Cache rows without a rotated part, from a projection without a query latent; every query has one key that stands
    out, far back, at a page's border, or its own."""
    from pilottai_amd import ops
    from pilottai_amd.ops.latent import latent_pad

    g, reqs, eps, Rp = gen(R + H), STEPS[step], 1e-3, latent_pad(R)
    T, m, dec, tile = fed_step(device, reqs, H, 1, 0, 0, tiles=256)
    pages = torch.full((700, Rp // 8, 16, 8), 9.0).to(dt)
    wc = torch.rand(R, generator=g) + 0.5
    x, q = torch.zeros(T, R + 40).to(dt), torch.zeros(T, H, Rp).to(dt)
    seqs = []
    for i, (c, n) in enumerate(reqs):
        a = torch.randn(c + n, R, generator=g).to(dt)
        rows = oracle.rms_norm(a.double(), wc.double(), eps)
        q0 = int(m["q_start"][i])
        x[q0:q0 + n, 16:16 + R] = a[c:]
        for t in range(c):  # what earlier steps left
            pages[int(m["block_table"][i, t // 16]), :, t % 16] = torch.cat([rows[t], torch.zeros(Rp - R)]).view(-1, 8).to(dt)
        for t in range(n):
            for h in range(H):
                far = [0, c + t, max(0, (c + t) // 16 * 16 - 1), (c + t) // 2][(t + h) % 4]
                q[q0 + t, h, :R] = (rows[far] * 12 / R + torch.randn(R, generator=g) * 0.3 / R ** 0.5).to(dt)
        seqs.append(rows)
    d = lambda t: t.to(device)  # noqa: E731
    pages = d(pages)
    ops.latent_cache(d(x)[:, 16:], 0, R, 0, None, d(wc), None, pages, Rp, m["positions"], m["slots"], None, eps)
    NB, mi = (dec * H + 15) // 16, m["items"].shape[0]
    out = torch.empty(T, H, Rp, dtype=dt, device=device)
    po, pm = torch.empty(mi * NB * 16 * Rp, device=device), torch.empty(mi * NB * 32, device=device)
    ops.latent_attention(out, po, pm, d(q), pages, m["items"], m["n_items"], *(m[k] for k in ("q_start", "q_len", "ctx_len", "block_table")),
                         1.0, 0, dec, tile, num_seqs=len(reqs))
    for i, (c, n) in enumerate(reqs):
        q0, rows = int(m["q_start"][i]), seqs[i]
        for h in range(H):
            full = torch.zeros(c + n, R, dtype=torch.float64)
            full[c:] = q[q0:q0 + n, h, :R].double()
            want = (oracle.causal_softmax(full @ rows.T) @ rows)[c:]
            torch.testing.assert_close(out[q0:q0 + n, h, :R].double().cpu(), want, **tol(dt, 2.0), msg=lambda s, i=i: f"request {i} {reqs[i]}: {s}")
    assert not out[:, :, R:].any()


@pytest.mark.parametrize("kind", ["plain", "rotated", "shared", "shared with a rotated part"])
@kinds
def test_latent_mixers(device, dt, kind):
    """The mixer alone, its own or another layer's cache, against keys and values written out per head."""
    from pilottai_amd.models.cache import StepMeta
    from pilottai_amd.models.hybrid import AttentionRoom, MixerBlock
    from pilottai_amd.models.latent import LatentAttention, LatentAttentionSpec
    from pilottai_amd.ops.latent import pad_to

    g, T, d, dev, eps, V = gen(5), 53, 72, torch.device(device), 1e-3, 70
    plain = dict(heads=6, dim=20, vdim=36, kv_rank=V, scale=0.5)
    turned = dict(heads=4, dim=40, vdim=24, kv_rank=V, scale=0.2, q_rank=28, rot_dim=12, rot_dims=12, rot_base=50.0)
    first, second = {"plain": (None, plain), "rotated": (None, turned), "shared": (plain, plain),
                     "shared with a rotated part": (turned, plain)}[kind]
    draw = lambda spec: {k: (torch.randn(s, generator=g) * (1.4 / s[-1] ** 0.5 if len(s) > 1 else 0.2) + (len(s) == 1)).to(BF16)  # noqa: E731
                         for k, s in spec.shapes(d).items()}
    make = lambda m, **kw: LatentAttentionSpec(**m, rot_pairs="rot_dim" in m, gate="rot_dim" not in m, **kw)  # noqa: E731
    h = torch.zeros(T, pad_to(d, 64)).to(dt)
    h[:, :d] = torch.randn(T, d, generator=g).to(dt)
    h0 = torch.zeros(T, pad_to(d, 64)).to(dt)  # the input of the layer that has the cache
    h0[:, :d] = torch.randn(T, d, generator=g).to(dt)
    iv = lambda *v: torch.tensor(v, dtype=torch.int32, device=dev)  # noqa: E731
    table = torch.tensor([[4, 0, 2, 3]], dtype=torch.int32)
    slots = torch.tensor([int(table[0, t // 16]) * 16 + t % 16 for t in range(T)], dtype=torch.int32)
    H = second["heads"]
    dec, tile = 16 // H, 128 // H
    items = [[0, b, min(tile, T - b) | 1 << 20, 0] for b in range(0, T, tile)]
    meta = StepMeta(iv(0), torch.arange(T, dtype=torch.int32, device=dev), slots.to(dev), iv(0), iv(T), iv(T), table.to(dev),
                    torch.tensor(items, dtype=torch.int32, device=dev), iv(len(items)), iv(0), iv(0), num_seqs=1)

    def oracle_of(m, w, x, c=None):
        w = {k: v.double() for k, v in w.items()}
        if "rot_dim" in m:
            return oracle.attend_latent_rotated(x, dict(m, rot={"base": m["rot_base"], "dims": m["rot_dims"]}), w, eps)
        c = oracle.latent(x, w, V, eps)[0] if c is None else c
        return oracle.attend_latent(x, c, m, w), c
    source, c, pages = None, None, None
    z = torch.zeros(len(items) * 64 * 512, device=dev)
    room = AttentionRoom(z, z, dec, tile, 0)
    for m, x, spec in ([(first, h0, make(first))] if first else []) + [(second, h, make(second, **({"kv_from": 0} if first else {})))]:
        w = draw(spec)
        cs = spec.angles(64).to(dev) if spec.rot_dim else None
        mixer = LatentAttention(spec, w, eps, dt, dev, cs, source)
        if pages is None:
            pages = torch.full((5, mixer.D // 8, 16, 8), 3.0, dtype=dt, device=dev)
        y = MixerBlock([mixer], dt, dev)(x.to(dev), meta, [(pages,)], room)[0]
        want, c = oracle_of(m, w, x[:, :d].double(), c)
        torch.testing.assert_close(y.double().cpu()[:, :d], want, **tol(dt, 2.0))
        source = mixer


# ---- gated linear attention ----------------------------------------------------------------------------
def memory_rows(g, T, H, N, V, r, spec, dt, spread):
    """Projection rows [q | k | v | a], padded, and what they hold."""
    np_, vp, rp = spec.padded
    x = torch.zeros(T, 2 * H * np_ + H * vp + rp + 8).to(dt)
    q, k, v, a = (torch.randn(T, *s, generator=g).to(dt) for s in ((H, N), (H, N), (H, V), (r,)))
    x[:, :H * np_].view(T, H, np_)[:, :, :N], x[:, H * np_:2 * H * np_].view(T, H, np_)[:, :, :N] = q, k
    x[:, 2 * H * np_:2 * H * np_ + H * vp].view(T, H, vp)[:, :, :V] = v
    x[:, 2 * H * np_ + H * vp:2 * H * np_ + H * vp + r] = a
    return x, q, k, v, a


def memory_weights(g, H, N, r, spec, dt, spread, bias):
    np_, _, rp = spec.padded
    a2, b = (torch.randn(H, N, r, generator=g) * spread / r ** 0.5).to(dt), bias + torch.randn(H, N, generator=g)
    full, fb = torch.zeros(H, np_, rp).to(dt), torch.zeros(H, np_)
    full[:, :N, :r], fb[:, :N] = a2, b
    return a2, b, full.view(H * np_, rp), fb.view(-1)


@kinds
@pytest.mark.parametrize("H,N,V,r,tau,spread,bias", [
    (3, 24, 20, 3, 16.0, 2.0, 0.0), (2, 64, 64, 16, 4.0, 1.0, 2.0), (1, 128, 150, 40, 16.0, 3.0, 1.0), (2, 48, 70, 16, 1.0, 4.0, 0.0),
    (2, 32, 16, 5, 0.05, 3.0, -2.0), (1, 160, 33, 7, 64.0, 6.0, 4.0), (2, 256, 40, 33, 8.0, 1.0, -1.0), (1, 16, 300, 64, 2.0, 8.0, 0.0)])
def test_linear_attention(device, dt, H, N, V, r, tau, spread, bias):
    """Sequences in portions of all lengths, several in a step, in slots that others have left; decays from none at
    all to states that are gone within a token."""
    from pilottai_amd import ops
    from pilottai_amd.models.hybrid import LinearAttentionSpec

    dev, g, rng = torch.device(device), gen(N + V), np.random.default_rng(N)
    spec = LinearAttentionSpec(H, N, V, tau, r)
    np_, vp, rp = spec.padded
    a2, b, a2p, bp = memory_weights(g, H, N, r, spec, dt, spread, bias)
    lengths = [230, 7, 75, 129]
    data, want = [], []
    for T in lengths:
        x, q, k, v, a = memory_rows(g, T, H, N, V, r, spec, dt, spread)
        z = torch.einsum("tr,hnr->thn", a.double(), a2.double()) + b.double()
        decay = torch.nn.functional.logsigmoid(z) / tau
        o, _ = oracle.linear_memory(q.double() * N ** -0.5, k.double(), v.double(), decay)
        data.append(x)
        want.append(o)
    cuts = [[64, 1, 9, 2, 66, 8, 80], [3, 4], [75], [128, 1]]
    state = torch.full((6, H, vp, np_), 1e4, device=dev)
    at, k = [0] * 4, [0] * 4
    iv = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)  # noqa: E731
    cols = (0, H * np_, 2 * H * np_, 2 * H * np_ + H * vp)
    while any(k[s] < len(cuts[s]) for s in range(4)):
        live = [s for s in range(4) if k[s] < len(cuts[s]) and (rng.random() < 0.7 or k[s] == 0)]
        if not live:
            continue
        ns = [cuts[s][k[s]] for s in live]
        starts = np.concatenate([[0], np.cumsum(ns)])
        T, pad = int(starts[-1]), int(rng.integers(0, 3))
        x, items = torch.zeros(T + pad, data[0].shape[1]).to(dt), []
        for i, s in enumerate(live):
            x[starts[i]:starts[i + 1]] = data[s][at[s]:at[s] + ns[i]]
            if ns[i] > ops.SCAN_MIN:
                items += [[i, c, min(ops.SCAN_CHUNK, ns[i] - c), 0] for c in range(0, ns[i], ops.SCAN_CHUNK)]
        y = torch.full((T + pad, H * vp + 16), 5.0, dtype=dt, device=dev)
        ops.linear_attention(x.to(dev), y[:, :H * vp], state, a2p.to(dev), bp.to(dev), iv(list(starts[:-1]) + [T, T]), iv(ns + [0, 0]),
                             iv([at[s] + n for s, n in zip(live, ns)] + [0, 0]), iv([4 - s for s in live] + [-1, -1]),
                             iv(items + [[0, 0, 0, 0]] * (100 - len(items))), iv([len(items)]), cols, N ** -0.5, 1.0 / tau, num_seqs=len(live))
        for i, s in enumerate(live):
            got = y[int(starts[i]):int(starts[i + 1]), :H * vp].double().cpu().view(-1, H, vp)
            ref = want[s][at[s]:at[s] + ns[i]]
            size = float(want[s].abs().max())
            torch.testing.assert_close(got[..., :V], ref, rtol=1e-2 if dt == BF16 else 1e-4, atol=(4e-3 if dt == BF16 else 2e-5) * size,
                                       msg=lambda m, s=s, n=ns[i]: f"sequence {s} at {at[s]}, {n} tokens: {m}")
            assert not got[..., V:].any()
            at[s] += ns[i]
            k[s] += 1
        assert (y[T:] == 5.0).all() and (y[:, H * vp:] == 5.0).all()
    assert (state[0] == 1e4).all() and (state[5] == 1e4).all()  # nobody's slots


@pytest.mark.gpu
@pytest.mark.parametrize("N,V,tau", [(64, 70, 16.0), (128, 32, 1.0), (96, 16, 4.0), (256, 64, 0.2)])
def test_linear_attention_keeps_the_state_in_fp32(gpu, N, V, tau):
    """The state that chunked portions leave equals that of single tokens to fp32's order, not bf16's."""
    from pilottai_amd import ops
    from pilottai_amd.models.hybrid import LinearAttentionSpec

    H, T, r, g = 3, 300, 16, gen(N)
    spec = LinearAttentionSpec(H, N, V, tau, r)
    np_, vp, _ = spec.padded
    _, _, a2, b = memory_weights(g, H, N, r, spec, BF16, 2.0, 1.0)
    x = memory_rows(g, T, H, N, V, r, spec, BF16, 2.0)[0].to(gpu)
    iv = lambda *v: torch.tensor(v, dtype=torch.int32, device=gpu)  # noqa: E731
    left = []
    for cuts in ([T], [130, 9, 161], [1] * T):
        state, at = torch.zeros(1, H, vp, np_, device=gpu), 0
        for n in cuts:
            items = [[0, c, min(64, n - c), 0] for c in range(0, n, 64)] if n > 8 else [[0, 0, 0, 0]]
            y = torch.empty(n, H * vp, dtype=BF16, device=gpu)
            ops.linear_attention(x[at:at + n], y, state, a2.to(gpu), b.to(gpu), iv(0), iv(n), iv(at + n), iv(0),
                                 torch.tensor(items, dtype=torch.int32, device=gpu), iv(len(items) if n > 8 else 0),
                                 (0, H * np_, 2 * H * np_, 2 * H * np_ + H * vp), N ** -0.5, 1.0 / tau, num_seqs=1)
            at += n
        left.append(state.cpu())
    for state in left[:2]:
        torch.testing.assert_close(state, left[2], rtol=1e-4, atol=1e-4 * float(left[2].abs().max()))


@kinds
@pytest.mark.parametrize("H,V,Vp", [(6, 20, 32), (8, 64, 64), (1, 16, 16), (5, 24, 32), (8, 256, 256)])
def test_norm_before_a_silu_gate(device, dt, H, V, Vp):
    from pilottai_amd import ops

    g, T, eps = gen(H * V), 11, 1e-3
    y, z = torch.randn(T, H * Vp + 24, generator=g).to(dt), torch.randn(T, H * Vp + 40, generator=g).to(dt)
    w, slots = torch.randn(V, generator=g).repeat(H), torch.arange(T, dtype=torch.int32)
    slots[4] = -1
    rows = y.to(device).clone()
    ops.gated_norm(rows[:, :H * Vp], z.to(device)[:, 8:], w.to(device), slots.to(device), H, V, Vp, H, eps, after="silu")
    o = rows.double().cpu()
    pick = lambda t: t.double()[:, :H * Vp].reshape(T, H, Vp)[:, :, :V]  # noqa: E731
    want = oracle.rms_norm(pick(y), w[:V].double(), eps).reshape(T, -1) * oracle.silu(pick(z[:, 8:]).reshape(T, -1))
    live = slots >= 0
    torch.testing.assert_close(pick(o).reshape(T, -1)[live], want[live], **tol(dt))
    assert not o[live][:, :H * Vp].view(-1, H, Vp)[:, :, V:].any() and torch.equal(o[:, H * Vp:], y.double()[:, H * Vp:])
