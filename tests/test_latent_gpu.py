"""Kernels of csrc/ops/{residual_norm, latent_cache, latent_attention, grouped_gemm}.hip against
plain fp32 formulas, in bf16 (MFMA) and fp32, at sizes that are not whole tiles."""
import math

import numpy as np
import pytest
import torch

pytestmark = pytest.mark.gpu
DTYPES = [torch.bfloat16, torch.float32]


def tol(dt):
    return dict(rtol=2e-2, atol=2e-2) if dt == torch.bfloat16 else dict(rtol=2e-5, atol=2e-5)


def norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("D,K,add", [(192, 1, None), (100, 3, "add"), (2048, 6, "add"), (50, 2, "set"), (4096, 1, None)])
def test_residual_norm(gpu, dt, D, K, add):
    from pilottai_amd import ops

    g = torch.Generator().manual_seed(D + K)
    T, V, ld, eps = 9, 31, (D + 63) // 64 * 64, 1e-4
    r, y = torch.randn(T, D, generator=g), torch.randn(T * K, ld, generator=g).to(dt)
    wp, wn = torch.rand(D, generator=g) + 0.5, torch.rand(D, generator=g) + 0.5
    emb, ids = torch.randn(V, D, generator=g).to(dt), torch.randint(0, V, (T,), generator=g, dtype=torch.int32)
    kw = dict(y=y, partials=K, y_scale=1 / K, w_post=wp)
    want = r + norm(y.float()[:, :D].view(T, K, D).sum(1) / K, wp, eps)
    if add == "add":
        want, kw = want + emb[ids.long()].float(), dict(kw, emb=emb, ids=ids, emb_add=True)
    elif add == "set":
        want, kw = emb[ids.long()].float(), dict(emb=emb, ids=ids)
    kw = {k: v.to(gpu) if torch.is_tensor(v) else v for k, v in kw.items()}
    rows = torch.tensor([3, 0, 3, 8], dtype=torch.int32)
    rg = r.to(gpu)
    out = torch.full((4, ld), 7.0, dtype=dt, device=gpu)
    ops.residual_norm(rg, eps, w_next=wn.to(gpu), out=out, rows=rows.to(gpu), **kw)  # leaves the residual alone
    torch.testing.assert_close(rg.cpu(), r, rtol=0, atol=0)
    torch.testing.assert_close(out.float().cpu()[:, :D], norm(want, wn, eps)[rows.long()], **tol(dt))
    assert not out[:, D:].any()
    out = torch.full((T, ld), 7.0, dtype=dt, device=gpu)
    ops.residual_norm(rg, eps, w_next=wn.to(gpu), out=out, **kw)
    torch.testing.assert_close(rg.cpu(), want, rtol=1e-5, atol=1e-5)
    torch.testing.assert_close(out.float().cpu()[:, :D], norm(want, wn, eps), **tol(dt))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T", [1, 40, 130])
@pytest.mark.parametrize("G,N,K", [(3, 48, 32), (5, 208, 96), (2, 512, 128)])
def test_head_gemm(gpu, dt, T, G, N, K):
    from pilottai_amd import ops

    g = torch.Generator().manual_seed(T + N)
    x, w = torch.randn(T, G * (K + 32), generator=g).to(dt), (torch.randn(G, N, K, generator=g) / math.sqrt(K)).to(dt)
    out = torch.full((T, G * (N + 16)), 5.0, dtype=dt, device=gpu)
    ops.head_gemm(x.to(gpu), K + 32, ops.pack_groups(w, dt).to(gpu), out, N + 16)
    o = out.float().cpu().view(T, G, N + 16)
    want = torch.einsum("tgk,gnk->tgn", x.float().view(T, G, K + 32)[:, :, :K], w.float())
    torch.testing.assert_close(o[:, :, :N], want, **tol(dt))
    assert (o[:, :, N:] == 5.0).all()


@pytest.mark.parametrize("dt,tm", [(torch.bfloat16, 16), (torch.bfloat16, 64), (torch.bfloat16, 256), (torch.float32, 16)])
@pytest.mark.parametrize("T,E,top,ff,D", [(1, 5, 2, 40, 96), (900, 4, 2, 72, 200), (600, 2, 2, 128, 256), (77, 7, 3, 96, 160), (300, 12, 1, 64, 64), (130, 70, 5, 32, 128)])
def test_table_experts(gpu, dt, tm, T, E, top, ff, D):
    from pilottai_amd import ops
    from pilottai_amd.ops.latent import pad_to

    g = torch.Generator().manual_seed(T * E)
    V, lim, fp = 50, 0.7, pad_to(ff, 128 if tm == 256 else 32)
    tabs = [torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(V)]).int() for _ in range(2)]
    ids = torch.randint(0, V, (T,), generator=g, dtype=torch.int32)
    slots = torch.arange(T, dtype=torch.int32)
    slots[T // 3: T // 3 + T // 8] = -1  # padding rows go through no expert
    cap = T * top // tm + min(E, T * top)
    desc = torch.tensor([[i * V * top, V, top, E, i * T * top, i * cap, cap, 0] for i in range(2)], dtype=torch.int32)
    order = torch.empty(2 * T * top, dtype=torch.int32, device=gpu)
    tiles = torch.empty(2 * cap, 4, dtype=torch.int32, device=gpu)
    nt = torch.empty(2, dtype=torch.int32, device=gpu)
    ops.table_route(torch.cat([t.reshape(-1) for t in tabs]).to(gpu), desc.to(gpu), desc, ids.to(gpu), slots.to(gpu), T,
                    tm, order, tiles, nt)
    DK, DN = (pad_to(D, 128),) * 2 if tm == 256 else (pad_to(D, 32), pad_to(D, 16))
    x = torch.randn(T, pad_to(D, 128), generator=g).to(dt)
    w1, w3 = [(torch.randn(E, ff, D, generator=g) / math.sqrt(D) * 1.5).to(dt) for _ in range(2)]
    w2 = (torch.randn(E, D, ff, generator=g) / math.sqrt(ff)).to(dt)
    z = lambda a, b: torch.zeros(E, a, b, dtype=dt)  # noqa: E731
    g1, g3, g2 = z(fp, DK), z(fp, DK), z(DN, fp)
    g1[:, :ff, :D], g3[:, :ff, :D], g2[:, :D, :ff] = w1, w3, w2
    p13 = ops.pack_groups(ops.interleave_gate_up(g1, g3), dt).to(gpu)
    p2 = ops.pack_groups(g2, dt).to(gpu)
    for i, tab in enumerate(tabs):
        act = torch.empty(T * top, fp, dtype=dt, device=gpu)
        y = torch.full((T * top, DN), 3.0, dtype=dt, device=gpu)
        sel = (tiles[i * cap:(i + 1) * cap], nt[i:i + 1], order[i * T * top:(i + 1) * T * top], T * top)
        ops.expert_gemm(x.to(gpu), p13, act, *sel, x_div=top, out_order=False, tm=tm, glu=(lim, 1.702, 1.0))
        ops.expert_gemm(act, p2, y, *sel, x_div=0, out_order=True, tm=tm)
        y = y.float().cpu().view(T, top, -1)[:, :, :D]
        assert (y[slots < 0] == 3.0).all()
        es = tab[ids.long()].long()
        for e in range(E):
            t, k = torch.nonzero((es == e) & (slots >= 0)[:, None], as_tuple=True)
            v = x[t, :D].float()
            a, u = (v @ w1[e].float().T).clamp(max=lim), (v @ w3[e].float().T).clamp(-lim, lim)
            torch.testing.assert_close(y[t, k], (a * torch.sigmoid(1.702 * a) * (u + 1)) @ w2[e].float().T, **tol(dt))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("NQ,R,r,rd,H", [(72, 104, 48, 48, 3), (50, 70, 24, 12, 5), (256, 512, 64, 64, 2)])
def test_latent_cache_and_query_rotation(gpu, dt, NQ, R, r, rd, H):
    from pilottai_amd import ops
    from pilottai_amd.ops import reference as ref
    from pilottai_amd.ops.latent import latent_pad, pad_to

    g = torch.Generator().manual_seed(R)
    T, Rp, rp, eps, base = 37, latent_pad(R), pad_to(r, 32), 1e-3, 900.0
    x = torch.randn(T, pad_to(NQ + R + r, 128), generator=g).to(dt)
    wq, wc = torch.rand(NQ, generator=g) + 0.5, torch.rand(R, generator=g) + 0.5
    pos = torch.arange(T, dtype=torch.int32) * 7 + 3
    slots = torch.randperm(5 * 16, generator=g)[:T].int()
    slots[5] = -1
    cs = ref.rope_cos_sin(400, rd, base)
    cq = torch.full((T, pad_to(NQ, 64)), 9.0, dtype=dt, device=gpu)
    pages = torch.full((5, (Rp + rp) // 8, 16, 8), 4.0, dtype=dt, device=gpu)
    ops.latent_cache(x.to(gpu), NQ, R, r, wq.to(gpu), wc.to(gpu), cq, pages, Rp, pos.to(gpu), slots.to(gpu), cs.to(gpu), eps)
    torch.testing.assert_close(cq.float().cpu()[:, :NQ], norm(x.float()[:, :NQ], wq, eps), **tol(dt))
    assert not cq[:, NQ:].any()

    def rot(v, p):  # [.., r]
        a = torch.tensor([p * base ** (-2.0 * i / rd) for i in range(rd // 2)], dtype=torch.float64)
        c, s = a.cos().float(), a.sin().float()
        u, w = v[..., :rd // 2], v[..., rd // 2:rd]
        return torch.cat([u * c - w * s, w * c + u * s, v[..., rd:]], -1)

    rows = pages.float().cpu().permute(0, 2, 1, 3).reshape(80, -1)
    for t in range(T):
        if slots[t] < 0:
            continue
        row = rows[slots[t]]
        torch.testing.assert_close(row[:R], norm(x[t].float()[NQ:NQ + R], wc, eps), **tol(dt))
        torch.testing.assert_close(row[Rp:Rp + r], rot(x[t].float()[NQ + R:NQ + R + r], int(pos[t])), **tol(dt))
        assert not row[R:Rp].any() and not row[Rp + r:].any()
    free = [s for s in range(80) if s not in slots.tolist()]
    assert (rows[free] == 4.0).all()
    # the queries' rotated part, beside their projection
    hs, N = 32 + rp, 48
    q, w = torch.randn(T, H * hs, generator=g).to(dt), (torch.randn(H, N, 32, generator=g) / 6).to(dt)
    dst = torch.full((T, H, N + rp + 16), 6.0, dtype=dt, device=gpu)
    ops.head_gemm(q.to(gpu), hs, ops.pack_groups(w, dt).to(gpu), dst.view(T, -1), N + rp + 16,
                  rot=(pos.to(gpu), cs.to(gpu), 32, r, rp))
    d = dst.float().cpu()
    assert (d[:, :, N + rp:] == 6.0).all() and not d[:, :, N + r:N + rp].any()
    torch.testing.assert_close(d[:, :, :N], torch.einsum("thk,hnk->thn", q.float().view(T, H, hs)[:, :, :32], w.float()), **tol(dt))
    for t in range(T):
        torch.testing.assert_close(d[t, :, N:N + r], rot(q[t].float().view(H, hs)[:, 32:32 + r], int(pos[t])), **tol(dt))


def fed_meta(gpu, H, reqs, split_target=384, window=0, nblocks=600, part=128, tiles=0):
    """Scheduler-built step: reqs [(cached tokens, new tokens)]; pages in scrambled order."""
    from pilottai_amd import _runtime

    group = min(H, 16)
    s = _runtime.Scheduler({"num_blocks": nblocks, "block_size": 16, "max_num_seqs": 16, "max_num_batched_tokens": 4096,
                            "max_model_len": 4096, "gqa_group": group, "kv_heads": 1, "att_qcols": 128,
                            "att_narrow_qcols": 128, "prefix_caching": False, "decode_part_target": split_target,
                            "att_max_keys": window, "att_min_part": part, "att_tile_target": tiles})
    L = s.layout()
    buf = np.zeros(L["total"], dtype=np.int32)
    junk = [(1000 + i, [1] * (16 * (1 + i % 3))) for i in range(8)]  # fragment the pool first
    s.schedule_fed(buf.ctypes.data, junk)
    s.commit(0, 0)
    for i in (1, 3, 4, 6):
        s.abort(1000 + i)
    for i, (c, _) in enumerate(reqs):
        if c:
            s.schedule_fed(buf.ctypes.data, [(i + 1, [1] * c)])
            s.commit(0, 0)
            if i < 4:
                s.abort([1000, 1002, 1005, 1007][i])
    T = s.schedule_fed(buf.ctypes.data, [(i + 1, [1] * n) for i, (_, n) in enumerate(reqs)])
    t = torch.from_numpy(buf)
    sl = lambda k, n: t[L[k]:L[k] + n].clone()  # noqa: E731
    ms, mb = L["max_seqs"], L["max_blocks"]
    m = dict(q_start=sl("q_start", ms), q_len=sl("q_len", ms), ctx_len=sl("ctx_len", ms),
             block_table=sl("block_table", ms * mb).view(ms, mb), items=sl("items", 4 * L["max_items"]).view(-1, 4),
             n_items=sl("n_items", 1))
    return T, m, 16 // group, 128 // group


def run_attention(gpu, dt, H, R, r, reqs, window, simple=False, split_target=384, seed=0, spike=None, **kw):
    from pilottai_amd import ops
    from pilottai_amd.ops.latent import latent_pad, pad_to

    g = torch.Generator().manual_seed(seed)
    Rp, rp = latent_pad(R), pad_to(r, 32)
    D = Rp + rp
    T, m, dec, tile = fed_meta(gpu, H, reqs, split_target, window, **kw)
    pages = torch.randn(600, D // 8, 16, 8, generator=g).to(dt)
    pages[:, R // 8:Rp // 8] = 0
    q = (torch.randn(T, H, D, generator=g) * 2).to(dt)
    if spike is not None:  # one key per query token answers loudly: it must be seen, or not, exactly
        spike(q, pages, m)
    NB, mi = (dec * H + 15) // 16, m["items"].shape[0]
    out = torch.full((T, H, Rp), 9.0, dtype=dt, device=gpu)
    po = torch.empty(mi * NB * 16 * Rp, dtype=torch.float32, device=gpu)
    pm = torch.empty(mi * NB * 32, dtype=torch.float32, device=gpu)
    mg = {k: v.to(gpu) for k, v in m.items()}
    scale = 1 / math.sqrt(R + r)
    ops.latent_attention(out, po, pm, q.to(gpu), pages.to(gpu), mg["items"], mg["n_items"], mg["q_start"],
                         mg["q_len"], mg["ctx_len"], mg["block_table"], scale, window, dec, tile, simple=simple)
    o = out.float().cpu()
    for i, (c, n) in enumerate(reqs):
        ctx, q0 = c + n, int(m["q_start"][i])
        rows = pages[m["block_table"][i, :(ctx + 15) // 16].long()].permute(0, 2, 1, 3).reshape(-1, D)[:ctx].float()
        sc = torch.einsum("thd,kd->htk", q[q0:q0 + n].float(), rows) * scale
        back = torch.arange(c, ctx)[:, None] - torch.arange(ctx)[None, :]
        sc = sc.masked_fill(~((back >= 0) & ((back < window) if window else True)), -math.inf)
        want = torch.einsum("htk,kd->thd", torch.softmax(sc, -1), rows[:, :Rp])
        torch.testing.assert_close(o[q0:q0 + n], want, **tol(dt), msg=lambda s, i=i: f"request {i} {reqs[i]}: {s}")


SHAPES = [(1, 32, 8), (3, 96, 24), (8, 100, 40), (16, 512, 64), (20, 256, 32), (40, 192, 64)]
STEPS = {"prompt": [(0, 75)], "decode": [(0, 1), (15, 1), (16, 1), (700, 1), (33, 1)], "two": [(130, 2), (0, 2)],
         "mixed": [(300, 1), (17, 40), (0, 3), (531, 130), (64, 1), (5, 2)]}


@pytest.mark.parametrize("window", [0, 1, 45, 128])
@pytest.mark.parametrize("step", list(STEPS))
@pytest.mark.parametrize("H,R,r", SHAPES)
def test_latent_attention_bf16(gpu, H, R, r, step, window):
    run_attention(gpu, torch.bfloat16, H, R, r, STEPS[step], window)


@pytest.mark.parametrize("window", [0, 45, 600])
@pytest.mark.parametrize("H,R,r", SHAPES)
def test_latent_attention_split_tiles(gpu, H, R, r, window):
    """Prompt portions cut over their keys: partitions of one item meet in the merge launch."""
    run_attention(gpu, torch.bfloat16, H, R, r, [(1500, 40), (900, 1), (0, 20), (700, 3)], window, tiles=64, part=256)
    tile = 128 // min(H, 16)  # and portions whose rest is as short as a decode row's tokens
    run_attention(gpu, torch.bfloat16, H, R, r, [(1500, tile + 1), (900, 2 * tile + 16 // min(H, 16))], window, tiles=64, part=256)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("window", [0, 45])
@pytest.mark.parametrize("step", ["decode", "mixed"])
def test_latent_attention_any_size(gpu, dt, window, step):
    run_attention(gpu, dt, 5, 72, 8, STEPS[step], window, simple=True)


@pytest.mark.parametrize("R", [32, 64, 96, 128, 192, 256, 384, 512, 600])
def test_latent_attention_every_width(gpu, R):
    run_attention(gpu, torch.bfloat16, 6, R, 64 if R % 64 else 32, [(200, 1), (20, 30)], 77)


@pytest.mark.parametrize("edge", ["first", "before"])
@pytest.mark.parametrize("reqs", [[(500, 1)], [(470, 1), (300, 60)], [(100, 2)]])
def test_latent_attention_window_edge(gpu, edge, reqs):
    """The oldest visible key (or the one just before it) outscores all others by far."""
    W = 91

    def spike(q, pages, m):
        for i, (c, n) in enumerate(reqs):
            k = c + n - W - (edge == "before")
            if k < 0:
                continue
            pg, off = int(m["block_table"][i, k // 16]), k % 16
            last = int(m["q_start"][i]) + n - 1
            q[last] = (3.0 * pages[pg, :, off].reshape(1, -1).float()).to(q.dtype)
    run_attention(gpu, torch.bfloat16, 4, 128, 32, reqs, W, spike=spike)
