"""The operations that the Salipel design brings, each alone (reference operations on the CPU; kernels on the GPU in
bf16 and fp32) against the plain functions of tests/salipel_oracle.py, at sizes that are not whole tiles."""
import math

import numpy as np
import pytest
import torch

import salipel_oracle as oracle
from test_hybrid_kernels import BF16, F32, SEQ, STEPS, fed_step, gen, kinds, pages_of, rows_of, tol


# ---- residual ----------------------------------------------------------------------------------------
@kinds
@pytest.mark.parametrize("D,K,weighted", [(72, 3, True), (256, 1, False), (50, 2, True), (2048, 6, True)])
def test_two_outputs_into_the_residual(device, dt, D, K, weighted):
    """One stream: x + m (weighted partials + a second output), and the next norm."""
    from pilottai_amd import ops

    g, T, ld, eps, mult = gen(D + K), 9, (D + 63) // 64 * 64, 1e-4, 0.6
    x, w = torch.randn(T, 1, D, generator=g), torch.rand(D, generator=g) + 0.5
    y, y2 = torch.randn(T * K, ld, generator=g).to(dt), torch.randn(T, ld + 64, generator=g).to(dt)
    yw = torch.rand(T, K, generator=g)
    d = lambda t: t.to(device)  # noqa: E731
    part = y.double()[:, :D].view(T, K, D)
    want = x.double()[:, 0] + mult * ((part * yw.double()[:, :, None]).sum(1) if weighted else part.sum(1)) + mult * y2.double()[:, :D]
    one, out, xg = torch.ones(1, device=device), torch.full((T, ld), 7.0, dtype=dt, device=device), d(x).clone()
    ops.hyper_norm(xg, eps, y=d(y), partials=K, y_weights=d(yw) if weighted else None, y2=d(y2)[:, :ld], mix=one.view(1, 1),
                   post=one * mult, pre=one, w_next=d(w), out=out)
    torch.testing.assert_close(xg.double().cpu()[:, 0], want, rtol=1e-5, atol=1e-4)
    torch.testing.assert_close(out.double().cpu()[:, :D], oracle.norm(want, w.double(), eps), **tol(dt))
    assert not out[:, D:].any()


# ---- rotation, heads and pages ---------------------------------------------------------------------------
@pytest.mark.parametrize("scaling", [None, (4.0, 1.0, 4.0, 64.0), (8.0, 1.0, 4.0, 8192.0), (3.0, 0.5, 9.0, 300.0), (2.0, 2.0, 2.5, 20.0)])
@pytest.mark.parametrize("dims,base", [(4, 10.0), (30, 300.0), (128, 500000.0)])
def test_angles(dims, base, scaling):
    from pilottai_amd import ops

    sc = dict(zip(("factor", "low", "high", "original"), scaling)) if scaling else None
    f = oracle.frequencies({"dims": dims, "base": base, "scaling": sc})
    a = torch.arange(5000, dtype=torch.float64)[:, None] * f
    torch.testing.assert_close(ops.angle_table(5000, dims, base, slow_waves=sc).double(), torch.cat([a.cos(), a.sin()], 1), rtol=0, atol=2e-6)


@kinds
@pytest.mark.parametrize("step", ["prompt", "decode", "mixed"])
@pytest.mark.parametrize("H,G,GV,dim,vdim,rd,qk,nv,tied", [
    (4, 2, 2, 40, 24, 20, True, False, False), (6, 1, 1, 64, 64, 16, True, False, True), (5, 5, 5, 33, 90, 0, False, True, False),
    (8, 4, 2, 24, 70, 24, True, False, False), (3, 3, 3, 128, 128, 128, True, True, False), (2, 1, 1, 250, 250, 100, True, False, True),
    (18, 2, 1, 8, 16, 4, True, True, False)])
def test_normed_heads(device, dt, H, G, GV, dim, vdim, rd, qk, nv, tied, step):
    """Head norms over the real dimensions, then the rotation (or none); values on the keys as projected."""
    from pilottai_amd import ops

    g, reqs, eps = gen(dim + vdim), STEPS[step], 1e-3
    T, m, _, _ = fed_step(device, reqs)
    dk, dv = ops.window_pad(dim, vdim)
    vcol = H * dk if tied else (H + G) * dk
    cols = (H + G) * dk + (0 if tied else GV * dv)
    wq, wk = (torch.cat([torch.rand(dim, generator=g) + 0.5, torch.zeros(dk - dim)]) for _ in range(2))
    new = lambda *s: torch.full(s, 4.0, dtype=dt)  # noqa: E731
    kp, vp = new(700, G, dk // 8, 16, 8).to(device), new(700, GV, dv // 8, 16, 8).to(device)
    none = torch.zeros(0, 1, 1, 8, dtype=dt, device=device)
    full, x = [], torch.zeros(T, cols + 8).to(dt)
    live = torch.cat([torch.ones((H + G) * dk).view(-1, dk).index_fill(1, torch.arange(dim, dk), 0.0).view(-1),
                      torch.ones(0 if tied else GV * dv).view(-1, dv).index_fill(1, torch.arange(vdim, dv), 0.0).view(-1)])
    for i, (c, n) in enumerate(reqs):
        r = (torch.randn(c + n, cols, generator=g) * live).to(dt)
        q0 = int(m["q_start"][i])
        x[q0:q0 + n, :cols] = r[c:]
        r = r.double()
        q, k = r[:, :H * dk].view(-1, H, dk), r[:, H * dk:(H + G) * dk].view(-1, G, dk)
        v = r[:, vcol:vcol + GV * dv].view(-1, GV, dv)
        part = lambda t, w: oracle.norm(t[..., :dim], w[:dim].double(), eps) if qk else t[..., :dim]  # noqa: E731
        q, k = part(q, wq), part(k, wk)
        if rd:
            q, k = (oracle.rotate(t, {"dims": rd, "base": 200.0}) for t in (q, k))
        v = v[..., :vdim]
        full.append((q, k, oracle.rms(v, eps) if nv else v))
    qo = torch.empty(T, H, dk, dtype=dt, device=device)
    d = lambda t: t.to(device)  # noqa: E731
    ops.paged_kv(d(x), None, qo, kp, vp, none, none, m["positions"], m["slots"], *(m[k] for k in SEQ),
                 d(ops.angle_table(1000, rd, 200.0)) if rd else None, 0, num_seqs=len(reqs), v_col=vcol if tied else -1,
                 q_norm=d(wq) if qk else None, k_norm=d(wk) if qk else None, norm_v=nv, dim=dim, vdim=vdim, eps=eps)
    for i, (c, n) in enumerate(reqs):
        q0, table = int(m["q_start"][i]), m["block_table"][i].cpu()
        for got, want, size in ((qo[q0:q0 + n], full[i][0], dim), (rows_of(kp.cpu(), table[:(c + n + 15) // 16], c + n)[c:], full[i][1], dim),
                                (rows_of(vp.cpu(), table[:(c + n + 15) // 16], c + n)[c:], full[i][2], vdim)):
            torch.testing.assert_close(got.double().cpu()[..., :size], want[c:], **tol(dt, 2.0))
            assert not got[..., size:].any()


# ---- attention -----------------------------------------------------------------------------------------
def run_attention(device, dt, H, G, GV, dk, dv, reqs, window=0, keep=0, chunk=0, bias=False, cap=0.0, sink=None, gate=False, gain=1.0,
                  wide_out=False, simple=False, seed=0, spread=1.0, spike=None, **kw):
    from pilottai_amd import ops

    g = gen(seed)
    T, m, dec, tile = fed_step(device, reqs, H // G, G, window + keep if window else chunk, 0, **kw)
    kp, vp = torch.full((700, G, dk // 8, 16, 8), 3.0), torch.full((700, GV, dv // 8, 16, 8), 50.0)
    q = (torch.randn(T, H, dk, generator=g) * spread).to(dt)
    z = torch.randn(T, H * dv + 40, generator=g).to(dt)
    seqs = []
    for i, (c, n) in enumerate(reqs):
        k, v = (torch.randn(c + n, heads, d, generator=g).to(dt).double() for heads, d in ((G, dk), (GV, dv)))
        if spike is not None:
            q0 = int(m["q_start"][i])
            spike(q[q0:q0 + n], k, v, c, n)
        seqs.append((k, v))
        pages_of(k.float(), m["block_table"][i], kp)
        pages_of(v.float(), m["block_table"][i], vp)
    NB, mi, scale = (dec * (H // G) + 15) // 16, m["items"].shape[0], 1 / math.sqrt(dk)
    whole = torch.full((T, H * dv + 64), 9.0, dtype=F32 if wide_out else dt, device=device)  # (heads inside longer rows)
    out = whole[:, 32:32 + H * dv].view(T, H, dv)
    po, pm = torch.empty(mi * G * NB * 16 * dv, device=device), torch.empty(mi * G * NB * 32, device=device)
    d = lambda t: t.to(dt).to(device)  # noqa: E731
    f = lambda t: t.float().to(device)  # noqa: E731
    none = torch.zeros(0, 1, 1, 8, dtype=dt, device=device)
    slopes = torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)])
    zg = z.to(device)[:, 8:8 + H * dv]
    ops.window_attention(out, po, pm, q.to(device), d(kp), d(vp), none, none, m["items"], m["n_items"], *(m[k] for k in SEQ), scale, window, 0,
                         f(sink) if sink is not None else None, dec, tile, mi, num_seqs=len(reqs), simple=simple, keep=keep, chunk=chunk,
                         slopes=f(slopes) if bias else None, cap=cap, gate=zg if gate else None, gain=gain)
    for i, (c, n) in enumerate(reqs):
        k, v = seqs[i]
        q0 = int(m["q_start"][i])
        for h in range(H):
            full = torch.zeros(c + n, dk, dtype=torch.float64)
            full[c:] = q[q0:q0 + n, h].double()
            want = oracle.attend(full, k[:, h * G // H], v[:, h * GV // H], scale, oracle.visible(c + n, window, keep, chunk),
                                 float(slopes[h]) if bias else 0.0, cap, sink[h].double() if sink is not None else None)[c:] * gain
            if gate:
                want = want * torch.sigmoid(z[q0:q0 + n, 8 + h * dv:8 + h * dv + dv].double())
            torch.testing.assert_close(out[q0:q0 + n, h].double().cpu(), want, **tol(dt), msg=lambda s, i=i: f"request {i} {reqs[i]}: {s}")
    assert (whole[:, :32] == 9.0).all() and (whole[:, 32 + H * dv:] == 9.0).all()


KINDS_OF = {
    "window": dict(window=45, keep=6, gate=True, gain=1.3), "long start": dict(window=20, keep=40), "one kept": dict(window=16, keep=1),
    "chunks": dict(chunk=48, bias=True, sink=True), "small chunks": dict(chunk=7, sink=True), "page chunks": dict(chunk=16, bias=True),
    "big chunks": dict(chunk=400, bias=True, sink=True), "cap": dict(cap=3.0, wide_out=True), "cap and bias": dict(cap=1.5, bias=True, gate=True),
    "plain": dict(gain=0.5)}


@kinds
@pytest.mark.parametrize("kind", list(KINDS_OF))
@pytest.mark.parametrize("step", list(STEPS))
@pytest.mark.parametrize("H,G,GV,dk,dv", [(2, 2, 2, 32, 32), (6, 2, 1, 64, 64), (4, 1, 1, 64, 32), (18, 2, 2, 128, 128)])
def test_attention(device, dt, H, G, GV, dk, dv, step, kind):
    if device == "cpu" and H not in (4, 6):
        pytest.skip("a selection on the CPU")
    kw = dict(KINDS_OF[kind])
    if kw.pop("sink", False):
        kw["sink"] = torch.randn(H, generator=gen(H)) * 2
    run_attention(device, dt, H, G, GV, dk, dv, STEPS[step], spread=3.0 if "cap" in kw else 1.0, **kw)


@pytest.mark.gpu
@pytest.mark.parametrize("kind", list(KINDS_OF))
@pytest.mark.parametrize("H,G,GV,dk,dv", [(6, 2, 1, 64, 64), (4, 1, 1, 64, 32), (16, 4, 4, 128, 128), (3, 3, 3, 256, 256)])
def test_attention_cut_over_keys(gpu, H, G, GV, dk, dv, kind):
    """Portions and decode rows whose keys are divided: empty partitions, kept tokens in the first one."""
    kw = dict(KINDS_OF[kind])
    if kw.pop("sink", False):
        kw["sink"] = torch.randn(H, generator=gen(H)) * 2
    run_attention(gpu, BF16, H, G, GV, dk, dv, [(1500, 40), (900, 1), (0, 20), (700, 3)], tiles=64, part=64, split=2000, **kw)


@pytest.mark.parametrize("group", [1, 2, 3, 4, 6, 16])
def test_partition_slots(group):
    """Portions cut over their keys: slots of their own for every partition, in a row: one where the portion's rest is no
    longer than a decode row's tokens (the kernels take it for one), else eight."""
    for tail in (1, 16 // group, 16 // group + 1):
        n = 2 * (128 // group) + tail
        _, m, dec, tile = fed_step("cpu", [(900, n), (700, 1), (1500, tail)], group, 1, part=64, tiles=64, split=2000)
        used, parts = set(), {}
        for seq, at, c, slot in m["items"][:int(m["n_items"])].tolist():
            nq, k = c & 0xff, c >> 20
            if k > 1:
                own = set(range(slot, slot + (1 if nq <= dec else 8)))
                assert not own & used and nq <= tile
                used |= own
                parts.setdefault((seq, at, nq, k), {})[c >> 8 & 0xfff] = slot
        for (_, _, nq, k), slots in parts.items():
            assert [slots[p] - slots[0] for p in range(k)] == [p * (1 if nq <= dec else 8) for p in range(k)]
        assert (0, n - tail, tail) in {key[:3] for key in parts} and max(used) < m["items"].shape[0]


@kinds
@pytest.mark.parametrize("H,G,GV,dk,dv", [(6, 1, 1, 64, 64), (4, 4, 2, 32, 64), (4, 1, 1, 64, 32)])
@pytest.mark.parametrize("mask", [{}, dict(window=300, keep=9), dict(chunk=1000)])
def test_a_cut_portion_with_a_short_rest(device, dt, H, G, GV, dk, dv, mask):
    tile = 128 // (H // G)
    run_attention(device, dt, H, G, GV, dk, dv, [(1200, tile + 1), (600, tile + 16 // (H // G)), (0, 2 * tile + 1)], tiles=64, part=64, split=2000, **mask)


@pytest.mark.gpu
@pytest.mark.parametrize("dk,dv", [(32, 32), (64, 32), (96, 96), (128, 64), (192, 128), (256, 256), (288, 320)])
def test_attention_every_width(gpu, dk, dv):
    run_attention(gpu, BF16, 6, 3, 3, dk, dv, [(200, 1), (20, 30)], window=77, keep=9, cap=4.0, gate=True)


@pytest.mark.gpu
@pytest.mark.parametrize("dt", [BF16, F32])
def test_any_size_kernel(gpu, dt):
    run_attention(gpu, dt, 4, 4, 2, 96, 32, STEPS["mixed"], window=45, keep=7, cap=4.0, bias=True, gate=True, simple=True)
    run_attention(gpu, dt, 6, 2, 2, 64, 64, STEPS["mixed"], chunk=33, bias=True, sink=torch.randn(6, generator=gen(1)), simple=True)


@kinds
@pytest.mark.parametrize("reqs", [[(500, 1)], [(470, 1), (300, 60)], [(101, 2)], [(0, 140)]])
@pytest.mark.parametrize("mask", [dict(window=91, keep=6), dict(window=64, keep=16), dict(window=30, keep=45), dict(chunk=96), dict(chunk=64), dict(chunk=21)])
def test_edges(device, dt, mask, reqs):
    """One key outscores all others by far for the last query: just inside and outside the window or chunk, the last
    kept and the first token that is not kept, the first of all."""
    def at(place):
        def spike(q, k, v, c, n):
            last = c + n - 1
            lo = last - last % mask["chunk"] if "chunk" in mask else last - mask["window"] + 1
            keep = mask.get("keep", 0)
            j = {"first": lo, "before": lo - 1, "kept": keep - 1, "unkept": keep, "start": 0}[place]
            if 0 <= j <= last:
                k[j] = (k[j] * 8).to(BF16).double()
                for h in range(q.shape[1]):
                    q[-1, h] = (k[j, h * k.shape[1] // q.shape[1]] / 4).to(q.dtype)
        return spike
    for place in ("first", "before", "kept", "unkept", "start"):
        run_attention(device, dt, 4, 2, 2, 64, 64, reqs, spike=at(place), **mask)


@kinds
def test_sinks(device, dt):
    """Sinks far below, at and far above the scores; a head's own number."""
    for sink in (-30.0, 0.0, 5.0, 40.0):
        s = torch.tensor([sink, sink + 1, -sink, 0.3])
        run_attention(device, dt, 4, 2, 2, 32, 32, [(40, 1), (0, 30)], chunk=25, sink=s)
        run_attention(device, dt, 4, 2, 2, 32, 32, [(300, 1), (0, 30)], sink=s, spread=6.0, part=64, split=2000)


@kinds
@pytest.mark.parametrize("G,R,D,vdim", [(2, 2, 64, 64), (1, 5, 96, 70), (3, 1, 32, 9), (2, 8, 256, 256)])
def test_head_difference(device, dt, G, R, D, vdim):
    from pilottai_amd import ops

    g, T, H, lam, diff, eps = gen(D), 7, G * R, 0.63, 0.35, 1e-3
    a, z = torch.randn(T, G, 2, R, D, generator=g), torch.randn(T, H * D + 24, generator=g).to(dt)
    a[..., vdim:] = 0
    rows = torch.full((T, H * D + 32), 9.0, dtype=dt, device=device)
    ops.head_difference(a.view(T, 2 * H, D).to(device), rows[:, 16:16 + H * D].view(T, H, D), z.to(device)[:, 8:8 + H * D], G, lam, 1 - diff, vdim, eps)
    x = a.double()[..., :vdim]
    want = oracle.differential(x[:, :, 0], x[:, :, 1], lam, diff, eps).reshape(T, H, vdim) * torch.sigmoid(z.double()[:, 8:8 + H * D].reshape(T, H, D)[..., :vdim])
    got = rows.double().cpu()
    torch.testing.assert_close(got[:, 16:16 + H * D].reshape(T, H, D)[..., :vdim], want, **tol(dt))
    assert not got[:, 16:16 + H * D].reshape(T, H, D)[..., vdim:].any() and (got[:, :16] == 9).all() and (got[:, 16 + H * D:] == 9).all()


# ---- matrix memory ---------------------------------------------------------------------------------------
def memory_rows(g, T, H, N, V, np_, vin, dt, gates=2.0):
    """Random projection rows [q | k | v | i | f] with padded heads, and their parts."""
    pad = lambda t, n: torch.nn.functional.pad(t, (0, n - t.shape[2])).reshape(T, -1)  # noqa: E731
    q, k, v = (torch.randn(T, H, n, generator=g).to(dt) for n in (N, N, V))
    z = (torch.randn(T, 2 * H, generator=g) * gates).to(dt)
    return torch.cat([pad(q, np_), pad(k, np_), pad(v, vin), z], 1), (q.double(), k.double(), v.double(), z.double())


def memory_want(parts, ib, fb, cap):
    q, k, v, z = parts
    H, N = q.shape[1:]
    i = cap * torch.tanh((z[:, :H] + ib.double()) / cap)
    f = torch.nn.functional.logsigmoid(cap * torch.tanh((z[:, H:] + fb.double()) / cap))
    return oracle.matrix_memory(q * N ** -0.5, k, v, i, f)


@kinds
@pytest.mark.parametrize("H,N,V,cap,gates", [(3, 32, 48, 15.0, 2.0), (2, 24, 20, 4.0, 6.0), (4, 64, 64, 12.0, 12.0), (1, 128, 250, 15.0, 2.0),
                                             (2, 96, 33, 8.0, 3.0), (1, 256, 64, 15.0, 1.0), (2, 160, 16, 15.0, 2.0)])
def test_matrix_memory(device, dt, H, N, V, cap, gates):
    """Requests in portions of all sizes, batched and reordered, against one pass over each whole sequence."""
    from pilottai_amd import ops
    from pilottai_amd.models.hybrid import MatrixMemorySpec

    g, dev = gen(H * V + N), torch.device(device)
    np_, vin, vs = MatrixMemorySpec(H, N, V, cap).padded
    cols, width = (0, H * np_, 2 * H * np_, 2 * H * np_ + H * vin, vin), 2 * H * np_ + H * vin + 2 * H
    ib, fb = torch.randn(H, generator=g), torch.linspace(-2.0, 6.0, H)
    plans = [[200, 1, 1, 2, 65], [1] * 12 + [8, 9, 64, 3, 100], [3, 130, 1, 7, 600]]
    data = [memory_rows(g, sum(p), H, N, V, np_, vin, dt, gates) for p in plans]
    want = [memory_want(parts, ib, fb, cap) for _, parts in data]
    state, top = torch.full((5, H, vs, np_), 1e4, device=dev), torch.full((5, H, vs), 1e4, device=dev)
    iv = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)  # noqa: E731
    at, k, rng = [0] * 3, [0] * 3, np.random.default_rng(0)
    while any(k[s] < len(plans[s]) for s in range(3)):
        live = [int(s) for s in rng.permutation(3) if k[s] < len(plans[s]) and rng.random() < 0.8]
        if not live:
            continue
        ns = [plans[s][k[s]] for s in live]
        starts = np.cumsum([0] + ns)
        T, pad = int(starts[-1]), int(rng.integers(0, 3))
        x, items = torch.zeros(T + pad, (width + 8) // 8 * 8).to(dt), []
        for i, s in enumerate(live):
            x[starts[i]:starts[i + 1], :width] = data[s][0][at[s]:at[s] + ns[i]]
            if ns[i] > ops.SCAN_MIN:
                items += [[i, b, min(ops.SCAN_CHUNK, ns[i] - b), 0] for b in range(0, ns[i], ops.SCAN_CHUNK)]
        y = torch.full((T + pad, H * vin + 16), 5.0, dtype=dt, device=dev)
        div = torch.full((T + pad, H), 5.0, device=dev)
        ops.matrix_memory(x.to(dev), y[:, :H * vin], div, state, top, ib.to(dev), fb.to(dev), iv(list(starts[:-1]) + [T, T]), iv(ns + [0, 0]),
                          iv([at[s] + n for s, n in zip(live, ns)] + [0, 0]), iv([4 - s for s in live] + [-1, -1]),
                          iv(items + [[0, 0, 0, 0]] * (100 - len(items))), iv([len(items)]), cols, V, cap, N ** -0.5, num_seqs=len(live))
        for i, s in enumerate(live):
            rows = slice(int(starts[i]), int(starts[i + 1]))
            got = y[rows, :H * vin].double().cpu().view(-1, H, vin)[..., :V] / div[rows].double().cpu()[..., None]
            ref = want[s][at[s]:at[s] + ns[i]]
            # (a quotient whose divisor may cancel: heads' rows relative to their size, all of them loosely)
            err = ((got - ref).pow(2).mean(-1).sqrt() / (ref.pow(2).mean(-1).sqrt() + 0.02)).reshape(-1)
            lim, mid = (0.15, 8e-3) if dt == BF16 else (3e-3, 2e-5)
            assert err.max() < lim and err.median() < mid, \
                f"sequence {s} at {at[s]}, {ns[i]} tokens: {float(err.max()):.2e}, median {float(err.median()):.2e}"
            at[s] += ns[i]
            k[s] += 1
        assert (y[T:] == 5.0).all() and (y[:, H * vin:] == 5.0).all() and (div[T:] == 5.0).all()
    assert (state[:2] == 1e4).all() and (top[:2] == 1e4).all()  # nobody's slots
    assert (top[2:, :, :V + 1] == top[2:, :, :1]).all()


@pytest.mark.gpu
@pytest.mark.parametrize("V", [32, 70])
def test_matrix_memory_keeps_the_state_in_fp32(gpu, V):
    """The state and maximum that chunked portions leave equal those of single tokens to fp32's order, not bf16's."""
    from pilottai_amd import ops
    from pilottai_amd.models.hybrid import MatrixMemorySpec

    H, N, T, cap = 3, 64, 300, 12.0
    np_, vin, vs = MatrixMemorySpec(H, N, V, cap).padded
    rows, _ = memory_rows(gen(5), T, H, N, V, np_, vin, BF16)
    x = torch.zeros(T, (rows.shape[1] + 8) // 8 * 8, dtype=BF16)
    x[:, :rows.shape[1]] = rows
    x, ib, fb = x.to(gpu), torch.zeros(H, device=gpu), torch.tensor([-1.0, 3.0, 8.0], device=gpu)
    iv = lambda *v: torch.tensor(v, dtype=torch.int32, device=gpu)  # noqa: E731
    left = []
    for cuts in ([T], [130, 9, 161], [1] * T):
        state, top, at = torch.zeros(1, H, vs, np_, device=gpu), torch.zeros(1, H, vs, device=gpu), 0
        for n in cuts:
            items = [[0, b, min(64, n - b), 0] for b in range(0, n, 64)] if n > 8 else [[0, 0, 0, 0]]
            y, div = torch.empty(n, H * vin, dtype=BF16, device=gpu), torch.empty(n, H, device=gpu)
            ops.matrix_memory(x[at:at + n], y, div, state, top, ib, fb, iv(0), iv(n), iv(at + n), iv(0), torch.tensor(items, dtype=torch.int32, device=gpu),
                              iv(len(items) if n > 8 else 0), (0, H * np_, 2 * H * np_, 2 * H * np_ + H * vin, vin), V, cap, N ** -0.5, num_seqs=1)
            at += n
        left.append((state.cpu(), top.cpu()))
    for state, top in left[:2]:
        torch.testing.assert_close(top[..., :V + 1], left[2][1][..., :V + 1], rtol=1e-5, atol=1e-4)
        torch.testing.assert_close(state, left[2][0], rtol=1e-4, atol=1e-4 * float(left[2][0].abs().max()))


@kinds
@pytest.mark.parametrize("H,V,Vp", [(6, 20, 32), (8, 64, 64), (1, 16, 16), (5, 24, 32), (8, 256, 256)])
def test_norm_before_the_gate(device, dt, H, V, Vp):
    from pilottai_amd import ops

    g, T, eps = gen(H * V), 11, 1e-3
    y, z = torch.randn(T, H * Vp + 24, generator=g).to(dt), torch.randn(T, H * Vp + 40, generator=g).to(dt)
    w, slots, div = torch.randn(H * V, generator=g), torch.arange(T, dtype=torch.int32), torch.rand(T, H, generator=g) * 3 + 0.01
    slots[4] = -1
    rows = y.to(device).clone()
    ops.gated_norm(rows[:, :H * Vp], z.to(device)[:, 8:], w.to(device), slots.to(device), H, V, Vp, H, eps, div=div.to(device), after="sigmoid")
    o = rows.double().cpu()
    pick = lambda t: t.double()[:, :H * Vp].reshape(T, H, Vp)[:, :, :V]  # noqa: E731
    want = oracle.rms(pick(y) / div.double()[:, :, None], eps).reshape(T, -1) * w.double() * torch.sigmoid(pick(z[:, 8:]).reshape(T, -1))
    live = slots >= 0
    torch.testing.assert_close(pick(o).reshape(T, -1)[live], want[live], **tol(dt))
    assert not o[live][:, :H * Vp].view(-1, H, Vp)[:, :, V:].any() and torch.equal(o[:, H * Vp:], y.double()[:, H * Vp:])


# ---- routing and experts ------------------------------------------------------------------------------
@kinds
@pytest.mark.parametrize("T", [1, 16, 17, 300])
@pytest.mark.parametrize("E,top,scale", [(8, 2, 1.3), (6, 6, 1.0), (64, 6, 2.5), (5, 1, 0.7), (160, 5, 1.0), (1, 1, 3.0)])
def test_softmax_route(device, dt, T, E, top, scale):
    """Choice by score + correction (of both signs), weights by the scores alone."""
    from pilottai_amd import ops

    g, D = gen(T + E), 72
    h, w, corr = torch.randn(T, 128, generator=g).to(dt), torch.zeros(1, (E + 15) // 16 * 16, 128).to(dt), torch.randn(E, generator=g) * 0.3
    h[:, D:] = 0
    w[0, :E, :D] = (torch.randn(E, D, generator=g) * 0.3).to(dt)
    slots = torch.arange(T, dtype=torch.int32)
    slots[T // 3:T // 3 + T // 8] = -1
    ints = lambda *n: torch.full(n, 0x3fffffff, dtype=torch.int32, device=device)  # noqa: E731
    weights, choice, order, tiles, n_tiles = torch.full((T, top), 9.0, device=device), ints(T * top), ints(T * top), ints(T * top // 16 + E, 4), ints(1)
    ops.score_route(h.to(device), ops.pack_groups(w, dt).to(device), slots.to(device), weights, choice, ints(T * top),
                    torch.zeros(E, dtype=torch.int32, device=device), order, tiles, n_tiles, E, top, 1, 1, 0, 16, softmax=True,
                    correction=corr.to(device), share=True, scale=scale)
    want = oracle.route(h.double(), w[0, :E].double(), corr.double(), {"top": top, "scale": scale})
    wt, ch, live = weights.double().cpu(), choice.cpu().view(T, top).long(), slots >= 0
    assert (ch[~live] == -1).all() and not wt[~live].any()
    got = torch.zeros(T, E, dtype=torch.float64)
    got[live] = got[live].scatter(1, ch[live], wt[live])
    same = ((got > 0) == (want > 0)).all(1) & live  # (a close call may fall differently)
    assert same.sum() >= 0.97 * live.sum()
    torch.testing.assert_close(got[same], want[same], rtol=2e-4, atol=1e-5)
    rows = [r for e, start, n, _ in tiles.cpu()[:int(n_tiles)].tolist() for r in order.cpu()[start:start + n].tolist()]
    assert sorted(rows) == [p for p in range(T * top) if bool(live[p // top])]


@kinds
@pytest.mark.parametrize("T", [8, 40])
@pytest.mark.parametrize("bits", [-1, 0x7fffffff, 0x7fc00000, -0x400000, 0x7f800000, -0x800000])
def test_routing_ignores_what_padding_holds(device, dt, T, bits):
    """Rows of no sequence hold any bits, NaNs among them: they are not placed and do not disturb the others."""
    from pilottai_amd import ops

    E, top, g = 8, 3, gen(7)
    h, w = torch.randn(T, 64, generator=g).to(dt), torch.randn(1, 16, 64, generator=g).to(dt)
    junk = torch.tensor([bits], dtype=torch.int32).view(F32) if dt == F32 else torch.tensor([bits >> 16], dtype=torch.int16).view(BF16)
    h[3:] = junk
    slots = torch.full((T,), -1, dtype=torch.int32)
    slots[:3] = torch.arange(3, dtype=torch.int32)
    ints = lambda *n: torch.full(n, 5, dtype=torch.int32, device=device)  # noqa: E731
    weights, choice, order, tiles, n_tiles = torch.full((T, top), 9.0, device=device), ints(T * top), ints(T * top), ints(T * top // 16 + E, 4), ints(1)
    ops.score_route(h.to(device), ops.pack_groups(w, dt).to(device), slots.to(device), weights, choice, ints(T * top),
                    torch.zeros(E, dtype=torch.int32, device=device), order, tiles, n_tiles, E, top, 1, 1, 0, 16, softmax=True, share=True)
    assert (choice.cpu()[3 * top:] == -1).all() and not weights.cpu()[3:].any()
    rows = [r for e, start, n, _ in tiles.cpu()[:int(n_tiles)].tolist() for r in order.cpu()[start:start + n].tolist()]
    assert sorted(rows) == list(range(3 * top))


@kinds
@pytest.mark.parametrize("T", [3, 90, 700])
@pytest.mark.parametrize("E,top,ff,d", [(6, 2, 40, 72), (4, 2, 128, 256), (9, 3, 200, 128)])
def test_experts_without_a_gate(device, dt, T, E, top, ff, d):
    from pilottai_amd.models.cache import StepMeta
    from pilottai_amd.models.hybrid import ScoredExperts, ScoredExpertsSpec
    from pilottai_amd.ops import pad_to

    g = gen(T + d)
    spec = ScoredExpertsSpec(experts=E, top=top, ff=ff, act=None, softmax=True, correction=True, share=True, scale=1.7)
    t = {k: (torch.randn(s, generator=g) / s[-1] ** 0.5 * 1.5).to(BF16) for k, s in spec.shapes(d).items()}
    t["correction"] = (torch.randn(E, generator=g) * 0.2).to(BF16)
    mod = ScoredExperts(spec, t, d, dt, torch.device(device))
    h = torch.zeros(T, pad_to(d, 64)).to(dt)
    h[:, :d] = torch.randn(T, d, generator=g).to(dt)
    meta = StepMeta(*([None] * 2), torch.arange(T, dtype=torch.int32, device=device), *([None] * 8))
    y, K, w, _ = mod(h.to(device), meta)
    got = (y.double().cpu().view(T, K, -1)[:, :, :d] * w.double().cpu()[:, :, None]).sum(1)
    want = oracle.feed_forward(h[:, :d].double(), {"kind": "moe", "router": {"top": top, "scale": 1.7}}, {k: v.double() for k, v in t.items()})
    ok = (got - want).abs().amax(1) < (0.06 if dt == BF16 else 2e-4) * float(want.abs().max())
    assert ok.float().mean() > 0.96  # (a close call swaps an expert)
