"""Every operation of ops/hybrid.py alone, reference operations (CPU) and kernels (GPU; bf16 and fp32),
against the plain functions of tests/mudepel_oracle.py, at sizes that are not whole tiles."""
import math

import numpy as np
import pytest
import torch

import mudepel_oracle as oracle

F32, BF16 = torch.float32, torch.bfloat16
KINDS = [("cpu", F32), pytest.param("cuda:0", F32, marks=pytest.mark.gpu), pytest.param("cuda:0", BF16, marks=pytest.mark.gpu)]
kinds = pytest.mark.parametrize("device,dt", KINDS)


def tol(dt, scale=1.0):
    return dict(rtol=2e-2, atol=2e-2 * scale) if dt == BF16 else dict(rtol=5e-5, atol=5e-5 * scale)


def gen(seed):
    return torch.Generator().manual_seed(seed)


# ---- residual ----------------------------------------------------------------------------------------
@kinds
@pytest.mark.parametrize("S,D,K,weighted", [(1, 72, 1, False), (2, 50, 3, True), (3, 160, 1, True), (4, 2048, 7, True), (5, 100, 2, False), (8, 4096, 1, False)])
def test_hyper_norm(device, dt, S, D, K, weighted):
    from pilottai_amd import ops

    g, T, ld, V, eps = gen(S * D), 9, (D + 63) // 64 * 64, 31, 1e-4
    x, y = torch.randn(T, S, D, generator=g), torch.randn(T * K, ld, generator=g).to(dt)
    mix, post, pre = torch.randn(S, S, generator=g), torch.randn(S, generator=g), torch.randn(S, generator=g)
    yw, bias, w = torch.rand(T, K, generator=g), torch.randn(D, generator=g), torch.randn(D, generator=g) * 0.2
    emb, ids = torch.randn(V, D, generator=g).to(dt), torch.randint(0, V, (T,), generator=g, dtype=torch.int32)
    d = lambda t: t.to(device)  # noqa: E731
    out = lambda n: torch.full((n, ld), 7.0, dtype=dt, device=device)  # noqa: E731
    # the start: every stream is the embedding row
    xs, o = torch.full((T, S, D), 3.0, device=device), out(T)
    ops.hyper_norm(xs, eps, emb=d(emb), ids=d(ids), pre=d(pre), w_next=d(1 + w), out=o)
    e = emb[ids.long()].double()
    torch.testing.assert_close(xs.double().cpu(), e[:, None].expand(-1, S, -1))
    torch.testing.assert_close(o.double().cpu()[:, :D], oracle.norm(float(pre.double().sum()) * e, w.double(), eps), **tol(dt))
    # a sublayer's output, then the next input
    part = y.double()[:, :D].view(T, K, D)
    yd = (part * yw.double()[:, :, None]).sum(1) + bias.double() if weighted else part.sum(1)
    hc = {"hc1.in": torch.zeros(S, dtype=torch.float64), "hc1.mix": mix.double(), "hc1.out": post.double()}
    want = oracle.hyper(x.double().permute(1, 0, 2), hc, 1, lambda _: yd)  # [S, T, D]
    h = oracle.norm((pre.double()[:, None, None] * want).sum(0), w.double(), eps)
    kw = dict(y=d(y), partials=K, y_weights=d(yw) if weighted else None, bias=d(bias) if weighted else None, mix=d(mix), post=d(post))
    rows = torch.tensor([3, 0, 3, 8], dtype=torch.int32)
    xg, o = d(x).clone(), out(4)
    ops.hyper_norm(xg, eps, pre=d(pre), w_next=d(1 + w), out=o, rows=d(rows), **kw)  # leaves the streams alone
    assert torch.equal(xg.cpu(), x)
    torch.testing.assert_close(o.double().cpu()[:, :D], h[rows.long()], **tol(dt))
    assert not o[:, D:].any()
    o = out(T)
    ops.hyper_norm(xg, eps, pre=d(pre), w_next=d(1 + w), out=o, **kw)
    torch.testing.assert_close(xg.double().cpu(), want.permute(1, 0, 2), rtol=1e-5, atol=1e-4)
    torch.testing.assert_close(o.double().cpu()[:, :D], h, **tol(dt))
    assert not o[:, D:].any()


@kinds
def test_softcap(device, dt):
    from pilottai_amd import ops

    x = (torch.randn(5, 301, generator=gen(1)) * 30).to(dt)
    y = ops.softcap(x.to(device).clone(), 290, 7.5).double().cpu()
    torch.testing.assert_close(y[:, :290], 7.5 * torch.tanh(x[:, :290].double() / 7.5), **tol(dt))
    assert torch.equal(y[:, 290:], x[:, 290:].double())


# ---- rotation ----------------------------------------------------------------------------------------
@pytest.mark.parametrize("scaling", [None, (2.5, 60.0, 4.0, 1.0), (8.0, 4096.0, 32.0, 1.0), (1.0, 100.0, 4.0, 2.0), (4.0, 16.0, 64.0, 32.0)])
@pytest.mark.parametrize("dims,base", [(4, 10.0), (32, 300.0), (80, 30000.0), (128, 500000.0)])
def test_angles(dims, base, scaling):
    from pilottai_amd import ops

    sc = dict(zip(("factor", "original", "fast", "slow"), scaling)) if scaling else None
    f, m = oracle.frequencies({"dims": dims, "base": base, "scaling": sc})
    a = torch.arange(5000, dtype=torch.float64)[:, None] * f
    torch.testing.assert_close(ops.angle_table(5000, dims, base, sc).double(), torch.cat([a.cos() * m, a.sin() * m], 1), rtol=0, atol=2e-6)


# ---- steps from the scheduler --------------------------------------------------------------------------
def fed_step(device, reqs, group=1, kv_heads=1, window=0, pool=0, blocks=700, part=128, tiles=0, split=384):
    """Scheduler-built step: reqs [(cached tokens, new tokens)]; pages in scrambled order."""
    from pilottai_amd import _runtime, ops

    s = _runtime.Scheduler({"num_blocks": blocks, "block_size": 16, "max_num_seqs": 16, "max_num_batched_tokens": 4096,
                            "max_model_len": 4096, "gqa_group": min(group, 16), "kv_heads": kv_heads, "att_qcols": 128,
                            "att_narrow_qcols": 128, "prefix_caching": False, "decode_part_target": split,
                            "att_max_keys": window, "att_pool": pool, "att_min_part": part, "att_tile_target": tiles,
                            "scan_chunk": ops.SCAN_CHUNK, "scan_min": ops.SCAN_MIN})
    L = s.layout()
    buf = np.zeros(L["total"], dtype=np.int32)
    s.schedule_fed(buf.ctypes.data, [(1000 + i, [1] * (16 * (1 + i % 3))) for i in range(8)])  # fragment the pool first
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
    sl = lambda k, n: t[L[k]:L[k] + n].clone().to(device)  # noqa: E731
    ms, mb = L["max_seqs"], L["max_blocks"]
    m = {k: sl(k, ms) for k in ("q_start", "q_len", "ctx_len", "state_slot", "scan_first")}
    m.update({k: sl(k, T) for k in ("positions", "slots")})
    m.update(block_table=sl("block_table", ms * mb).view(ms, mb), items=sl("items", 4 * L["max_items"]).view(-1, 4),
             n_items=sl("n_items", 1), scan_items=sl("scan_items", 4 * L["max_scan"]).view(-1, 4), n_scan=sl("n_scan", 1))
    return T, m, 16 // min(group, 16), 128 // min(group, 16)


SEQ = ("q_start", "q_len", "ctx_len", "block_table")
STEPS = {"prompt": [(0, 75)], "decode": [(0, 1), (15, 1), (16, 1), (700, 1), (33, 1)], "two": [(130, 2), (0, 2)],
         "mixed": [(300, 1), (17, 40), (0, 3), (531, 130), (64, 1), (5, 2)]}


def pages_of(rows, table, pages):
    """rows [n, G, D] -> their places in pages [blocks, G, D/8, 16, 8]."""
    for t in range(rows.shape[0]):
        pages[int(table[t // 16]), :, :, t % 16] = rows[t].view(rows.shape[1], -1, 8)


def rows_of(pages, table, n):
    G, d8 = pages.shape[1:3]
    return pages[table.long()].permute(0, 3, 1, 2, 4).reshape(-1, G, d8 * 8)[:n]


def pool_place(b, P):
    page = (b * P + P - 1) // 16
    return page, b - page * 16 // P


@kinds
@pytest.mark.parametrize("step", ["prompt", "two", "mixed"])
@pytest.mark.parametrize("H,G,dk,dv,rd,P,bias", [(4, 2, 32, 64, 32, 5, True), (3, 3, 64, 32, 20, 16, True), (6, 1, 96, 96, 96, 24, False), (2, 2, 32, 32, 4, 1, True), (5, 5, 128, 128, 128, 12, True), (2, 1, 32, 32, 16, 0, False)])
def test_paged_kv(device, dt, H, G, dk, dv, rd, P, bias, step):
    from pilottai_amd import ops

    g, reqs, rot = gen(dk + P), STEPS[step], {"dims": rd, "base": 200.0}
    T, m, _, _ = fed_step(device, reqs)
    cols = (H + G) * dk + G * dv
    per = ops.pooled_per_page(P)
    new = lambda *s: torch.full(s, 4.0, dtype=dt)  # noqa: E731
    kp, vp = new(700, G, dk // 8, 16, 8), new(700, G, dv // 8, 16, 8)
    pk, pv = (new(700, per, G, dk), new(700, per, G, dv)) if P else (new(0, 1, G, dk), new(0, 1, G, dv))
    b = torch.randn(cols, generator=g) if bias else None
    full, x = [], torch.zeros(T, cols + 8).to(dt)
    for i, (c, n) in enumerate(reqs):  # a whole sequence's rows; those of earlier steps are in its pages
        r = torch.randn(c + n, cols, generator=g).to(dt)
        x[int(m["q_start"][i]):int(m["q_start"][i]) + n, :cols] = r[c:]
        r = r.double() + (b.double() if bias else 0)
        q, k, v = r[:, :H * dk].view(-1, H, dk), r[:, H * dk:(H + G) * dk].view(-1, G, dk), r[:, (H + G) * dk:].view(-1, G, dv)
        q, k = oracle.rotate(q, rot), oracle.rotate(k, rot)
        full.append((q, k, v))
        pages_of(k[:c].to(dt), m["block_table"][i], kp)
        pages_of(v[:c].to(dt), m["block_table"][i], vp)
    kp, vp, pk, pv = (t.to(device) for t in (kp, vp, pk, pv))
    qo = torch.empty(T, H, dk, dtype=dt, device=device)
    ops.paged_kv(x.to(device), b.to(device) if bias else None, qo, kp, vp, pk, pv, m["positions"], m["slots"],
                 *(m[k] for k in SEQ), ops.angle_table(1000, rd, 200.0).to(device), P, num_seqs=len(reqs))
    written = set()
    for i, (c, n) in enumerate(reqs):
        q, k, v = full[i]
        q0, table = int(m["q_start"][i]), m["block_table"][i].cpu()
        torch.testing.assert_close(qo[q0:q0 + n].double().cpu(), q[c:], **tol(dt))
        for pages, want in ((kp, k), (vp, v)):
            torch.testing.assert_close(rows_of(pages.double().cpu(), table[:(c + n + 15) // 16], c + n), want, **tol(dt))
        for blk in range(c // P, (c + n) // P) if P else ():
            page, sub = pool_place(blk, P)
            written.add((int(table[page]), sub))
            for pooled, want in ((pk, k), (pv, v)):
                torch.testing.assert_close(pooled[int(table[page]), sub].double().cpu(), want[blk * P:blk * P + P].mean(0), **tol(dt))
    assert len(written) == sum((c + n) // P - c // P for c, n in reqs) if P else True
    left = torch.ones(pk.shape[:2], dtype=torch.bool)
    for p, s in written:
        left[p, s] = False
    assert (pk.cpu()[left] == 4.0).all() and (pv.cpu()[left] == 4.0).all()


# ---- attention -----------------------------------------------------------------------------------------
def run_attention(device, dt, H, G, dk, dv, reqs, W, P, sink=1.0, simple=False, seed=0, gain=1.0, spike=None, **kw):
    from pilottai_amd import ops

    g, per = gen(seed), ops.pooled_per_page(P)
    T, m, dec, tile = fed_step(device, reqs, H // G, G, W, P, **kw)
    kp, vp = torch.zeros(700, G, dk // 8, 16, 8), torch.zeros(700, G, dv // 8, 16, 8)
    pk, pv = (torch.full((700, per, G, d), 50.0) for d in (dk, dv))  # (blocks that are not seen must not be read as keys)
    q = (torch.randn(T, H, dk, generator=g) * gain).to(dt)
    seqs = []
    for i, (c, n) in enumerate(reqs):
        k, v = (torch.randn(c + n, G, d, generator=g).to(dt).double() for d in (dk, dv))
        if spike is not None:
            spike(q[int(m["q_start"][i]):int(m["q_start"][i]) + n], k, v, c, n)
        seqs.append((k, v))
        table = m["block_table"][i]
        pages_of(k.float(), table, kp)
        pages_of(v.float(), table, vp)
        for b in range((c + n) // P if P else 0):
            page, sub = pool_place(b, P)
            pk[int(table[page]), sub], pv[int(table[page]), sub] = (t[b * P:b * P + P].mean(0).float() for t in (k, v))
    NB, mi, scale = (dec * (H // G) + 15) // 16, m["items"].shape[0], 1 / math.sqrt(dk)
    out = torch.full((T, H, dv), 9.0, dtype=dt, device=device)
    po, pm = torch.empty(mi * G * NB * 16 * dv, device=device), torch.empty(mi * G * NB * 32, device=device)
    d = lambda t: t.to(dt).to(device)  # noqa: E731
    ops.window_attention(out, po, pm, q.to(device), d(kp), d(vp), d(pk), d(pv), m["items"], m["n_items"], *(m[k] for k in SEQ),
                         scale, W, P, torch.full((H,), math.log(sink), device=device) if sink else None, dec, tile, mi, num_seqs=len(reqs), simple=simple)
    for i, (c, n) in enumerate(reqs):
        k, v = seqs[i]
        q0 = int(m["q_start"][i])
        for h in range(H):
            whole = torch.zeros(c + n, dk, dtype=torch.float64)
            whole[c:] = q[q0:q0 + n, h].double()
            want = oracle.pooled_attention(whole, k[:, h * G // H], v[:, h * G // H], scale, W, P, sink)[c:]
            torch.testing.assert_close(out[q0:q0 + n, h].double().cpu(), want, **tol(dt), msg=lambda s, i=i: f"request {i} {reqs[i]}: {s}")


SHAPES = [(1, 1, 32, 32), (6, 2, 64, 32), (3, 3, 96, 96), (8, 1, 128, 64), (20, 1, 64, 64)]
MASKS = [(0, 0), (1, 0), (45, 0), (45, 12), (128, 16), (16, 5), (33, 50), (7, 1)]


@kinds
@pytest.mark.parametrize("W,P", MASKS)
@pytest.mark.parametrize("step", list(STEPS))
@pytest.mark.parametrize("H,G,dk,dv", SHAPES)
def test_window_attention(device, dt, H, G, dk, dv, step, W, P):
    if device == "cpu" and (H, W) not in ((6, 45), (6, 0), (3, 16)):
        pytest.skip("a selection on the CPU")
    run_attention(device, dt, H, G, dk, dv, STEPS[step], W, P)


@pytest.mark.gpu
@pytest.mark.parametrize("W,P", [(0, 0), (45, 4), (600, 12)])
@pytest.mark.parametrize("H,G,dk,dv", SHAPES)
def test_window_attention_split_tiles(gpu, H, G, dk, dv, W, P):
    """Prompt portions and decode rows cut over their keys and blocks: partitions meet in the merge launch."""
    run_attention(gpu, BF16, H, G, dk, dv, [(1500, 40), (900, 1), (0, 20), (700, 3)], W, P, tiles=64, part=256, split=2000)


@pytest.mark.gpu
@pytest.mark.parametrize("dk,dv", [(32, 32), (64, 32), (64, 64), (96, 96), (128, 64), (128, 128), (192, 128), (192, 192), (256, 256), (288, 320)])
def test_window_attention_every_width(gpu, dk, dv):
    run_attention(gpu, BF16, 6, 3, dk, dv, [(200, 1), (20, 30)], 77, 9)


@pytest.mark.gpu
@pytest.mark.parametrize("dt", [BF16, F32])
def test_window_attention_any_size_kernel(gpu, dt):
    run_attention(gpu, dt, 5, 5, 96, 32, STEPS["mixed"], 45, 7, simple=True)


@kinds
@pytest.mark.parametrize("sink", [0.0, 1.0])
def test_window_attention_sink(device, dt, sink):
    """Scores near 0 (the sink has the weight of a key) and far below and above it."""
    for gain in (0.0, 1.0, 12.0):
        run_attention(device, dt, 2, 1, 32, 32, [(40, 1), (0, 30)], 20, 6, sink=sink, gain=gain)

    def below(q, k, v, c, n):  # every score is about -20: without the sink the weights sum to 1, with it to nearly 0
        q[:] = torch.ones_like(q) * 4
        k[:] = -k.abs() - 0.5
    run_attention(device, dt, 2, 1, 32, 32, [(40, 1), (0, 30)], 20, 6, sink=sink, spike=below)


@kinds
@pytest.mark.parametrize("reqs", [[(500, 1)], [(470, 1), (300, 60)], [(101, 2)], [(0, 140)]])
@pytest.mark.parametrize("W,P", [(91, 12), (64, 16), (30, 45)])
def test_window_attention_edges(device, dt, W, P, reqs):
    """One key outscores all others by far, for the last query: the oldest of the window, the one just before
    it (seen through its block or not at all), and keys of the newest seen and the first unseen block."""
    def at(place):
        def spike(q, k, v, c, n):
            last = c + n - 1
            nb = max(0, last - W + 1) // P
            j = {"first": last - W + 1, "before": last - W, "block": nb * P - 1, "unseen": nb * P, "far": P // 2}[place]
            if 0 <= j <= last:
                k[j] = (k[j] * 8).to(BF16).double()
                for h in range(q.shape[1]):
                    q[-1, h] = (k[j, h * k.shape[1] // q.shape[1]] / 4).to(q.dtype)
        return spike
    for place in ("first", "before", "block", "unseen", "far"):
        run_attention(device, dt, 4, 2, 64, 64, reqs, W, P, spike=at(place))


# ---- state-space layers ---------------------------------------------------------------------------------
@kinds
@pytest.mark.parametrize("H,V,N,G,taps", [(4, 16, 32, 2, 4), (3, 32, 64, 1, 2), (6, 80, 96, 3, 6), (2, 64, 128, 2, 4), (1, 128, 256, 1, 8)])
def test_state_scan(device, dt, H, V, N, G, taps):
    """Requests in portions of all sizes, batched and reordered, against one pass over each whole sequence."""
    from pilottai_amd import ops

    g, dev = gen(H * V), torch.device(device)
    inner, bc, n_seq = H * V, G * N, 3
    C, cols = inner + 2 * bc, 2 * inner + 2 * bc + H
    tp, rows = ops.conv_taps(taps), ops.conv_taps(taps) - 1 + ops.SCAN_MIN
    conv, cb = torch.randn(C, taps, generator=g) * 0.5, torch.randn(C, generator=g) * 0.2
    dt_bias, a, d = torch.randn(H, generator=g) - 2, torch.linspace(0.02, 3.0, H), torch.randn(H, generator=g)
    plans = [[200, 1, 1, 2, 65], [1] * 12 + [8, 9, 64, 3, 100], [3, 130, 1, 7, 2, 2, 2]]
    seqs = [torch.randn(sum(p), cols, generator=g).to(dt) for p in plans]
    want = []
    for r in seqs:
        T = len(r)
        z, xbc, raw = torch.split(r.double(), [inner, C, H], 1)
        u = oracle.silu(oracle.causal_conv(xbc, conv.double(), cb.double())).to(dt).double()
        x, B, Cm = torch.split(u, [inner, bc, bc], 1)
        share = lambda y: y.reshape(T, G, N).repeat_interleave(H // G, 1)  # noqa: E731, B023
        step = torch.nn.functional.softplus(raw + dt_bias.double(), threshold=1e9)
        want.append(oracle.state_scan(x.reshape(T, H, V), share(B), share(Cm), step, -a.double(), d.double()).reshape(T, inner))
    state = torch.full((5, H, V, N), 1e4, device=dev)  # (a sequence that starts overwrites what its slot held)
    ring = torch.full((5, rows, C), 1e3, dtype=dt, device=dev)
    w = torch.cat([torch.zeros(C, tp - taps), conv], 1).T.contiguous()
    iv = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)  # noqa: E731
    f = lambda t: t.float().to(dev)  # noqa: E731
    at, k = [0] * n_seq, [0] * n_seq
    rng = np.random.default_rng(0)
    while any(k[s] < len(plans[s]) for s in range(n_seq)):
        live = [int(s) for s in rng.permutation(n_seq) if k[s] < len(plans[s]) and (rng.random() < 0.8)]
        if not live:
            continue
        ns = [plans[s][k[s]] for s in live]
        starts = np.cumsum([0] + ns)
        T, pad = int(starts[-1]), int(rng.integers(0, 3))
        proj = torch.zeros(T + pad, (cols + 7) // 8 * 8).to(dt)
        items, first = [], []
        for i, s in enumerate(live):
            proj[starts[i]:starts[i + 1], :cols] = seqs[s][at[s]:at[s] + ns[i]]
            first.append(len(items) if ns[i] > ops.SCAN_MIN else -1)
            if ns[i] > ops.SCAN_MIN:
                items += [[i, b, min(ops.SCAN_CHUNK, ns[i] - b), 0] for b in range(0, ns[i], ops.SCAN_CHUNK)]
        y = torch.full((T + pad, (inner + 63) // 64 * 64), 5.0, dtype=dt, device=dev)
        # two rows of no sequence behind, as in a captured step
        ops.state_scan(proj.to(dev), y, state, ring, f(w), f(cb), f(dt_bias), f(a), f(d), iv(list(starts[:-1]) + [T, T]),
                       iv(ns + [0, 0]), iv([at[s] + n for s, n in zip(live, ns)] + [0, 0]), iv([4 - s for s in live] + [-1, -1]),
                       iv(first + [-1, -1]), iv(items + [[0, 0, 0, 0]] * (100 - len(items))), iv([len(items)]), G, num_seqs=len(live))
        for i, s in enumerate(live):
            got, ref = y[starts[i]:starts[i + 1], :inner].double().cpu(), want[s][at[s]:at[s] + ns[i]]
            torch.testing.assert_close(got, ref, **tol(dt, float(ref.abs().mean()) + 0.1), msg=lambda e, s=s: f"sequence {s} at {at[s]}, {plans[s][k[s]]} tokens: {e}")
            at[s] += ns[i]
            k[s] += 1
        assert (y[T:] == 5.0).all()
    assert (state[:2] == 1e4).all() and (ring[:2] == 1e3).all()  # nobody's slots


@pytest.mark.gpu
def test_state_scan_keeps_the_state_in_fp32(gpu):
    """The state a chunked portion leaves equals the one that single tokens leave to fp32's order, not bf16's."""
    from pilottai_amd import ops

    H, V, N, G, T = 2, 32, 64, 1, 192
    g, C = gen(5), 2 * 32 + 2 * 64
    cols = H * V + C + H
    proj = torch.randn(T, (cols + 7) // 8 * 8, generator=g).to(BF16).to(gpu)
    w, cb = torch.randn(4, C, generator=g).to(gpu), torch.zeros(C, device=gpu)
    bias, a, d = torch.full((H,), -3.0, device=gpu), torch.tensor([0.01, 0.5], device=gpu), torch.ones(H, device=gpu)
    iv = lambda *v: torch.tensor(v, dtype=torch.int32, device=gpu)  # noqa: E731
    states = []
    for cuts in ([T], [1] * T):
        state, ring = torch.zeros(1, H, V, N, device=gpu), torch.zeros(1, 11, C, dtype=BF16, device=gpu)
        at = 0
        for n in cuts:
            items = [[0, b, min(64, n - b), 0] for b in range(0, n, 64)] if n > 8 else [[0, 0, 0, 0]]
            y = torch.empty(n, H * V, dtype=BF16, device=gpu)
            ops.state_scan(proj[at:at + n], y, state, ring, w, cb, bias, a, d, iv(0), iv(n), iv(at + n), iv(0),
                           iv(0 if n > 8 else -1), torch.tensor(items, dtype=torch.int32, device=gpu), iv(len(items) if n > 8 else 0), G, num_seqs=1)
            at += n
        states.append(state.cpu())
    torch.testing.assert_close(states[0], states[1], rtol=1e-4, atol=1e-4 * float(states[1].abs().max()))


@kinds
@pytest.mark.parametrize("H,V,Vp,parts", [(6, 20, 32, 2), (8, 64, 64, 8), (4, 16, 16, 1), (5, 24, 32, 5), (3, 48, 48, 4), (64, 64, 64, 8)])
def test_gated_norm(device, dt, H, V, Vp, parts):
    from pilottai_amd import ops

    g, T, eps, ld = gen(H * V), 11, 1e-3, (H * Vp + 63) // 64 * 64
    y, z = torch.randn(T, ld, generator=g).to(dt), torch.randn(T, H * Vp + 40, generator=g).to(dt)
    w, slots = torch.randn(H * V, generator=g), torch.arange(T, dtype=torch.int32)
    slots[4] = -1
    o = ops.gated_norm(y.to(device).clone(), z.to(device), w.to(device), slots.to(device), H, V, Vp, parts, eps).double().cpu()
    pick = lambda t: t.double()[:, :H * Vp].view(T, H, Vp)[:, :, :V].reshape(T, -1)  # noqa: E731
    v = (pick(y) * oracle.silu(pick(z))).reshape(T, parts, -1)
    live = slots >= 0
    torch.testing.assert_close(pick(o)[live], (oracle.rms(v, eps).reshape(T, -1) * w.double())[live], **tol(dt))
    assert not o[live][:, H * Vp:].any() and not o[live][:, :H * Vp].view(-1, H, Vp)[:, :, V:].any()


# ---- routing and feed-forwards ------------------------------------------------------------------------------
@kinds
@pytest.mark.parametrize("T", [1, 16, 17, 300])
@pytest.mark.parametrize("E,top,groups,keep,always", [(8, 2, 1, 1, 0), (6, 2, 3, 2, 1), (64, 6, 8, 4, 1), (12, 12, 2, 2, 3), (5, 1, 5, 1, 0), (160, 5, 4, 1, 2), (1, 1, 1, 1, 1), (70, 3, 35, 2, 0)])
def test_score_route(device, dt, T, E, top, groups, keep, always):
    from pilottai_amd import ops

    g, D, tm, KA = gen(T + E), 72, 16 if T < 300 else 64, top + always
    h, w = torch.randn(T, 128, generator=g).to(dt), torch.zeros(1, (E + 15) // 16 * 16, 128).to(dt)
    h[:, D:] = 0
    w[0, :E, :D] = (torch.randn(E, D, generator=g) * 0.3).to(dt)
    slots = torch.arange(T, dtype=torch.int32)
    slots[T // 3:T // 3 + T // 8] = -1
    ints = lambda *n: torch.full(n, -7, dtype=torch.int32, device=device)  # noqa: E731
    cap = T * KA // tm + min(E + always, T * KA)
    weights, choice, rank, order, tiles, n_tiles = torch.full((T, KA), 9.0, device=device), ints(T * KA), ints(T * KA), ints(T * KA), ints(cap, 4), ints(1)
    ops.score_route(h.to(device), ops.pack_groups(w, dt).to(device), slots.to(device), weights, choice, rank,
                    torch.zeros(E + always, dtype=torch.int32, device=device), order, tiles, n_tiles, E, top, groups, keep, always, tm)
    want = oracle.route(h.double(), w[0, :E].double(), {"experts": E, "top": top, "groups": {"count": groups, "keep": keep}})
    wt, ch = weights.double().cpu(), choice.cpu().view(T, KA).long()
    live = slots >= 0
    assert (ch[~live] == -1).all() and not wt[~live].any()
    got = torch.zeros(T, E + always, dtype=torch.float64)
    got[live] = got[live].scatter(1, ch[live], wt[live])
    full = torch.cat([want, torch.ones(T, always, dtype=torch.float64)], 1)
    # (a close call may fall differently: its weights are then nearly equal)
    same = ((got > 0) == (full > 0)).all(1) & live
    assert same.sum() >= 0.97 * live.sum()
    torch.testing.assert_close(got[same], full[same], rtol=1e-4, atol=1e-5)
    # every live (token, choice) once, sorted by expert in tiles of at most tm
    seen, order, nxt = [], order.cpu(), 0
    for e, start, n, _ in tiles.cpu()[:int(n_tiles)].tolist():
        assert 1 <= n <= tm and start == nxt
        nxt += n
        rows = order[start:start + n].tolist()
        assert all(int(ch.view(-1)[r]) == e for r in rows)
        seen += rows
    assert sorted(seen) == [p for p in range(T * KA) if bool(live[p // KA])]


@kinds
@pytest.mark.parametrize("T", [3, 90, 700])
@pytest.mark.parametrize("name,p,d", [("groups", {"experts": 6, "top": 2, "ff": 40, "groups": 3, "keep": 2, "shared_ff": 56}, 72),
                                      ("whole tiles", {"experts": 4, "top": 2, "ff": 128, "groups": 2, "keep": 1, "shared_ff": 128}, 256),
                                      ("no shared", {"experts": 9, "top": 3, "ff": 33}, 50)])
def test_scored_experts_module(device, dt, T, name, p, d):
    from pilottai_amd.models.cache import StepMeta
    from pilottai_amd.models.hybrid import ScoredExperts, ScoredExpertsSpec
    from pilottai_amd.ops import pad_to

    g, spec = gen(T + d), ScoredExpertsSpec(**p)
    t = {k: (torch.randn(s, generator=g) / s[1] ** 0.5 * 1.5).to(BF16) for k, s in spec.shapes(d).items()}
    mod = ScoredExperts(spec, t, d, dt, torch.device(device))
    h = torch.zeros(T, pad_to(d, 64)).to(dt)
    h[:, :d] = torch.randn(T, d, generator=g).to(dt)
    meta = StepMeta(*([None] * 2), torch.arange(T, dtype=torch.int32, device=device), *([None] * 8))
    y, K, w, _ = mod(h.to(device), meta)
    got = (y.double().cpu().view(T, K, -1)[:, :, :d] * w.double().cpu()[:, :, None]).sum(1)
    r = {"experts": spec.experts, "top": spec.top, "groups": {"count": spec.groups, "keep": spec.keep}}
    want = oracle.experts(h[:, :d].double(), {"router": r, "shared": bool(spec.shared_ff)}, {k: v.double() for k, v in t.items()})
    ok = (got - want).abs().amax(1) < (0.06 if dt == BF16 else 2e-4) * float(want.abs().max())
    assert ok.float().mean() > 0.96  # (a close call swaps an expert)


@kinds
@pytest.mark.parametrize("T", [3, 90, 700])
@pytest.mark.parametrize("d,ff", [(72, 56), (256, 384), (50, 130)])
def test_gated_mlp_module(device, dt, T, d, ff):
    from pilottai_amd.models.hybrid import DenseSpec, GatedMLP
    from pilottai_amd.ops import pad_to

    g, spec = gen(T + d), DenseSpec(ff)
    t = {k: (torch.randn(s, generator=g) / s[1] ** 0.5 * 1.5).to(BF16) for k, s in spec.shapes(d).items()}
    mod = GatedMLP(spec, t, d, dt, torch.device(device))
    h = torch.zeros(T, pad_to(d, 64)).to(dt)
    h[:, :d] = torch.randn(T, d, generator=g).to(dt)
    y = mod(h.to(device), None)[0].double().cpu()[:, :d]
    want = oracle.gated(h[:, :d].double(), {k: v.double() for k, v in t.items()}, "", oracle.gelu_tanh)
    torch.testing.assert_close(y, want, **tol(dt, 2.0))
