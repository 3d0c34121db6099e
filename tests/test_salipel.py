"""The Salipel model in the engine against the plain implementation of tests/salipel_oracle.py: whole prompts,
portions, batches, reused pages and state slots, edges of windows and chunks, long decoding and generation, on the CPU
(reference operations, fp32) and on the GPU (the kernels, fp32 and bf16)."""
import copy
import json
import os
import subprocess

import numpy as np
import pytest
import torch

import salipel_oracle as oracle

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DEVICES = ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)]
KINDS = [("cpu", "float32"), pytest.param("cuda:0", "float32", marks=pytest.mark.gpu),
         pytest.param("cuda:0", "bfloat16", marks=pytest.mark.gpu)]


def sizes(heads, kv, dim, vdim, scale):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale or 1.2 / dim ** 0.5}


def rot(dims, base=300.0, scaling=None):
    r = {"base": base, "dims": dims}
    return dict(r, scaling=dict(zip(("factor", "low", "high", "original"), scaling))) if scaling else r


def chunked(heads, kv, dim, vdim, size, scale=None):
    return "attention", dict(sizes(heads, kv, dim, vdim, scale), mask={"size": size})


def twice(heads, kv, dim, vdim, dims, cap, diff, scaling=None, scale=None):
    return "attention_2", dict(sizes(heads, kv, dim, vdim, scale), rot=rot(dims, 500.0, scaling), softcap=cap, diff=diff)


def both(left, memory, window, keep=0, dims=None, scaling=None, scales=(1.0, 1.0), scale=None):
    """left: (heads, KV heads, dim); memory: (heads, dim, vdim, gate cap)."""
    h, kv, n = left
    mask = dict({"size": window}, **({"keep_first": keep} if keep else {}))
    return "parallel", {"left": dict(sizes(h, kv, n, n, scale), rot=rot(dims or n, 300.0, scaling), mask=mask),
                        "right": dict(zip(("heads", "dim", "vdim", "gate_cap"), memory)), "left_scale": scales[0], "right_scale": scales[1]}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, scale=1.0):
    return {"kind": "moe", "router": {"experts": experts, "top": top, "scale": scale}, "expert": {"ff": ff}}


def design(layers, width=72, vocab=101, eps=1e-4, mult=0.8):
    return {"architecture": "Salipel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult,
            "layers": [{"type": m[0], "mixer": m[1], "mlp": p} for m, p in layers]}


DESIGNS = {
    # every mixer with every feed-forward, unequal everything
    "varied": design([(both((6, 2, 40), (3, 24, 20, 9.0), 19, 5, dims=12, scaling=(3.0, 1.0, 4.0, 60.0), scales=(0.7, 1.6)), moe(6, 2, 40, 2.5)),
                      (chunked(3, 1, 40, 24, 25), dense(56)), (twice(4, 2, 24, 40, 20, 7.0, 0.3), moe(5, 1, 24, 0.6)),
                      (both((3, 3, 36), (1, 40, 50, 15.0), 33, 40), dense(100)), (chunked(4, 4, 16, 36, 64), None),
                      (twice(3, 1, 36, 20, 36, 20.0, 0.6, scaling=(2.0, 0.5, 8.0, 30.0)), dense(33))]),
    # recurrence first, whole tiles, a chunk of whole pages, no kept tokens, weights of 1
    "memory_first": design([(both((4, 4, 32), (4, 32, 32, 5.0), 32), dense(128)), (chunked(8, 2, 64, 64, 32), moe(8, 3, 64)),
                            (twice(8, 8, 32, 64, 32, 30.0, 0.5), None)], width=128, vocab=257, mult=1.0),
    # no recurrent layer: prefixes may be cached
    "attention_only": design([(twice(2, 1, 20, 33, 10, 3.0, 0.2), moe(9, 4, 20, 1.3)), (chunked(5, 5, 24, 10, 7), dense(33)),
                              (chunked(2, 1, 96, 96, 200), moe(4, 4, 32))], width=50, vocab=64),
    # side by side only; a wide group, a wide memory, many kept tokens
    "parallel_only": design([(both((18, 1, 8), (2, 130, 70, 12.0), 40, 3, dims=4), moe(12, 5, 70, 1.9)), (both((2, 1, 64), (5, 16, 9, 3.0), 11, 50), None)],
                            width=96, vocab=130, mult=0.5),
    "wide": design([(chunked(3, 3, 130, 70, 50), None), (twice(6, 3, 130, 200, 100, 15.0, 0.45), dense(40)), (both((2, 2, 250), (1, 256, 100, 15.0), 25, 13, dims=250), moe(3, 2, 130))],
                   width=200, vocab=90, mult=1.2),
}


def weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    d, V = cfg["width"], cfg["vocab"]
    t = {}

    def lin(name, n, k, gain=1.0):
        t[name] = (torch.randn(n, k, generator=g) * gain / k ** 0.5).to(torch.bfloat16)

    def around(name, shape, mean, dev):
        t[name] = (mean + dev * torch.randn(shape, generator=g)).to(torch.bfloat16)

    def attention(p, m, maps=1, values=True, gate=True, norms=True):
        lin(p + "q", m["heads"] * maps * m["dim"], d)
        lin(p + "k", m["kv_heads"] * maps * m["dim"], d)
        if values:
            lin(p + "v", m["kv_heads"] * m["vdim"], d)
        lin(p + "o", d, m["heads"] * m["vdim"])
        if gate:
            lin(p + "g", m["heads"] * m["vdim"], d, 1.5)
        for k in ("q.norm", "k.norm") if norms else ():
            around(p + k, m["dim"], 1.0, 0.2)

    t["embed"], t["head"] = (torch.randn(V, d, generator=g).to(torch.bfloat16) for _ in range(2))
    t["head"] = (t["head"].float() / d ** 0.5).to(torch.bfloat16)
    for i, L in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", L["mixer"], L["mlp"]
        around(p + "norm1", d, 1.0, 0.2)
        if L["type"] == "attention":
            attention(p + "mix.", m, gate=False, norms=False)
            around(p + "mix.sink", m["heads"], 0.0, 1.0)
        elif L["type"] == "attention_2":
            attention(p + "mix.", m, maps=2)
            for k in ("lq1", "lk1", "lq2", "lk2"):
                around(p + "mix." + k, m["dim"], 0.0, 0.25)
        else:
            r = m["right"]
            attention(p + "mix.left.", m["left"], values=False)
            for k, n in (("q", r["heads"] * r["dim"]), ("k", r["heads"] * r["dim"]), ("v", r["heads"] * r["vdim"]), ("g", r["heads"] * r["vdim"])):
                lin(p + "mix.right." + k, n, d)
            lin(p + "mix.right.o", d, r["heads"] * r["vdim"])
            around(p + "mix.right.norm", r["heads"] * r["vdim"], 1.0, 0.2)
            for k, lo, hi in (("i", -1.0, 2.0), ("f", 0.5, 5.0)):
                lin(p + "mix.right." + k, r["heads"], d, 1.5)
                t[p + f"mix.right.{k}.b"] = torch.linspace(lo, hi, r["heads"]).to(torch.bfloat16)  # short and long memories
        if f and f["kind"] == "dense":
            for k, n, j in (("gate", f["ff"], d), ("up", f["ff"], d), ("down", d, f["ff"])):
                lin(p + "mlp." + k, n, j, 1.3)
        elif f:
            E = f["router"]["experts"]
            lin(p + "mlp.router", E, d, 2.0)
            around(p + "mlp.correction", E, 0.0, 0.1)
            for e in range(E):
                lin(f"{p}mlp.e{e}.up", f["expert"]["ff"], d)
                lin(f"{p}mlp.e{e}.down", d, f["expert"]["ff"], 0.4)  # (a close call in bf16 swaps an expert: of limited weight)
    around("final.norm", d, 1.0, 0.2)
    return t


@pytest.fixture(scope="session")
def folder(tmp_path_factory):
    from safetensors.torch import save_file

    made = {}

    def make(name):
        if name not in made:
            p = tmp_path_factory.mktemp(name)
            (p / "config.json").write_text(json.dumps(DESIGNS[name]))
            save_file(weights(DESIGNS[name]), str(p / "model.safetensors"))
            made[name] = str(p)
        return made[name]
    return make


_want = {}


def expect(folder, name, ids):
    """Oracle logits of one sequence (a longer one's rows serve its prefixes: the design is causal)."""
    key = (name, tuple(ids))
    for (n, k), v in _want.items():
        if n == name and k[:len(ids)] == key[1]:
            return v[:len(ids)]
    _want[key] = oracle.forward(DESIGNS[name], oracle.read_checkpoint(folder(name)), ids)
    return _want[key]


def tokens(name, n, seed=1):
    return torch.randint(0, DESIGNS[name]["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def engine(folder, name, device, dtype, **kw):
    from pilottai_amd.engine.engine import EngineConfig, LLMEngine

    kw = dict(dict(max_num_seqs=4, max_num_batched_tokens=256, max_model_len=256, num_kv_blocks=40, exact_kv_blocks=True,
                   prefix_caching=False, use_graphs=False), **kw)
    return LLMEngine(EngineConfig(model=folder(name), dtype=dtype, **kw), device=device)


def close(got, want, dtype, what=""):
    got, want = got.double().cpu(), want.double()
    err = (got - want).pow(2).mean(1).sqrt() / want.std()
    # bf16: a router's close call swaps an expert on single rows, and the recurrent states carry it on, hence
    # the median; the kernels' own tests hold every row, and fp32 holds the whole structure to 5e-4
    lim, mid = (5e-4, 1e-4) if dtype == "float32" else (1.0, 0.08)
    assert err.max() < lim and (len(err) < 16 or err.median() < mid), \
        f"{what}: row {int(err.argmax())} of {len(err)} is off by {float(err.max()):.2e}, median {float(err.median()):.2e}"


def feed(eng, rid, ids, cuts):
    out, lo = [], 0
    for n in cuts:
        out.append(eng.feed_step([(rid, ids[lo:lo + n], list(range(n)))]))
        lo += n
    assert lo == len(ids)
    return torch.cat(out)


@pytest.mark.parametrize("device,dtype", KINDS)
@pytest.mark.parametrize("name", list(DESIGNS))
def test_prompt(folder, name, device, dtype):
    eng = engine(folder, name, device, dtype)
    ids = tokens(name, 150)
    close(feed(eng, 1, ids, [150]), expect(folder, name, ids), dtype)


@pytest.mark.parametrize("device,dtype", KINDS)
@pytest.mark.parametrize("cuts", [[2] * 75, [17] * 8 + [14], [1] * 150, [16, 16, 3, 2, 32, 64, 17], [9, 8, 10, 65, 58], [120] + [1] * 30])
def test_portions_and_decoding(folder, device, dtype, cuts):
    eng = engine(folder, "varied", device, dtype)
    ids = tokens("varied", 150)
    close(feed(eng, 1, ids, cuts), expect(folder, "varied", ids), dtype)


@pytest.mark.parametrize("device,dtype", KINDS)
@pytest.mark.parametrize("name", [n for n in DESIGNS if n != "varied"])
def test_portions_of_every_design(folder, name, device, dtype):
    eng = engine(folder, name, device, dtype)
    ids = tokens(name, 150)
    close(feed(eng, 1, ids, [7, 2, 1, 1, 30, 3, 66, 2, 8] + [1] * 30), expect(folder, name, ids), dtype)


@pytest.mark.parametrize("device,dtype", KINDS)
@pytest.mark.parametrize("name", ["varied", "memory_first"])
def test_residual_after_every_layer(folder, name, device, dtype):
    eng = engine(folder, name, device, dtype)
    ids = tokens(name, 29)
    want, got = [], []
    oracle.forward(DESIGNS[name], oracle.read_checkpoint(folder(name)), ids, layers=want)
    eng.feed_step([(1, ids, [0])], residuals=got)
    assert len(got) == len(want) == len(DESIGNS[name]["layers"])
    for j, (g, w) in enumerate(zip(got, want)):
        close(g[:len(ids)], w, dtype, f"layer {j}")


@pytest.mark.parametrize("device,dtype", KINDS)
@pytest.mark.parametrize("name", ["varied", "parallel_only"])
def test_mixed_batches_and_reused_pages_and_slots(folder, name, device, dtype):
    """Unequal requests join, pause, leave and take over freed pages and slots; each must equal itself alone."""
    eng = engine(folder, name, device, dtype, num_kv_blocks=19)
    rng = np.random.default_rng(3)
    live, rid, done = {}, 0, 0
    while done < 9:
        while len(live) < 4 and rid < 9:
            n = int(rng.integers(1, 100))
            if sum((len(v[0]) + 15) // 16 for v in live.values()) + (n + 15) // 16 > 19:
                break
            live[rid] = [tokens(name, n, 50 + rid), 0]
            rid += 1
        entries = []
        for r, (ids, at) in live.items():
            if len(live) > 1 and rng.random() < 0.25:
                continue
            n = min(len(ids) - at, int(rng.choice([1, 1, 1, 2, 5, 9, 16, 40, 70])))
            entries.append((r, ids[at:at + n], list(range(n))))
        if not entries:
            continue
        rng.shuffle(entries)
        out, k = eng.feed_step(entries), 0
        for r, toks, _ in entries:
            ids, at = live[r]
            close(out[k:k + len(toks)], expect(folder, name, ids)[at:at + len(toks)], dtype, f"request {r} at {at}")
            k += len(toks)
            live[r][1] += len(toks)
            if live[r][1] == len(ids):
                eng.release_fed(r)
                del live[r]
                done += 1
    assert eng.sched.num_free_blocks == 19 and eng.sched.num_free_states == 4


@pytest.mark.parametrize("device,dtype", KINDS)
def test_batch_does_not_change_a_request(folder, device, dtype):
    name = "memory_first"
    ids = tokens(name, 60)
    alone = feed(engine(folder, name, device, dtype), 1, ids, [44] + [1] * 16)
    eng = engine(folder, name, device, dtype)
    other = tokens(name, 200, 9)
    eng.feed_step([(7, other[:90], [])])
    rows, at = [], 90
    for lo, n in [(0, 44)] + [(44 + i, 1) for i in range(16)]:
        rows.append(eng.feed_step([(7, other[at:at + 3], []), (1, ids[lo:lo + n], list(range(n)))]))
        at += 3
    close(torch.cat(rows), alone.cpu(), dtype)


@pytest.mark.parametrize("device,dtype", KINDS)
@pytest.mark.parametrize("name", ["varied", "attention_only"])
def test_long_decoding_past_every_window(folder, name, device, dtype):
    eng = engine(folder, name, device, dtype)
    ids = tokens(name, 200)
    close(feed(eng, 1, ids, [3] + [1] * 197), expect(folder, name, ids), dtype)


@pytest.mark.parametrize("device", DEVICES)
def test_a_slot_starts_empty(folder, device):
    """A sequence in a slot that another has left, and one whose first portions are single tokens."""
    name = "parallel_only"
    eng = engine(folder, name, device, "float32", max_num_seqs=1, num_kv_blocks=16)
    for seed, cuts in ((1, [70]), (2, [1] * 20), (3, [2] * 10), (4, [12])):
        ids = tokens(name, sum(cuts), seed)
        close(feed(eng, seed, ids, cuts), expect(folder, name, ids), "float32", f"seed {seed}")
        eng.release_fed(seed)


def one_layer(tmp_path, cfg, device, change=None):
    from safetensors.torch import save_file

    t = weights(cfg)
    if change:
        change(t)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(t, str(tmp_path / "model.safetensors"))
    return engine(lambda _: str(tmp_path), "", device, "float32", max_num_batched_tokens=128)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind,size,keep", [("window", 21, 6), ("window", 16, 0), ("window", 5, 17), ("window", 40, 1), ("chunk", 30, 0), ("chunk", 16, 0), ("chunk", 7, 0)])
def test_what_a_position_sees(device, tmp_path, kind, size, keep):
    """One attention layer: another token changes the last position's logits exactly if it lies in the window or chunk
    or among the kept first ones, in whole prompts, in portions and in decoding."""
    mixer = both((2, 1, 16), (1, 8, 8, 4.0), size, keep, scales=(1.0, 0.0)) if kind == "window" else chunked(2, 1, 16, 16, size)
    cfg = design([(mixer, None)], width=32, vocab=40)
    eng = one_layer(tmp_path, cfg, device, lambda t: t.update({"l0.mix.sink": torch.full((2,), -2.0).to(torch.bfloat16)}) if kind == "chunk" else None)
    n = 86
    ids = torch.randint(0, 40, (n,), generator=torch.Generator().manual_seed(size)).tolist()
    last = n - 1
    lo = last - size + 1 if kind == "window" else last - last % size
    base = oracle.forward(cfg, oracle.read_checkpoint(str(tmp_path)), ids)[-1]
    for j in {lo, lo - 1, 0, keep - 1, keep, last - 1}:
        if not 0 <= j < last:
            continue
        seen = j >= lo or j < keep
        other = list(ids)
        other[j] = (other[j] + 1) % 40
        for cuts in ([n], [64] + [1] * 22, [2] * 43, [30, 37, 19]):
            got = feed(eng, 2, other, cuts)[-1].double().cpu()
            eng.release_fed(2)
            # (a distance bias makes the oldest key of a chunk faint, not gone)
            assert ((got - base).abs().max() > 2e-5) == seen, (j, seen, cuts[:3], float((got - base).abs().max()))


@pytest.mark.parametrize("device", DEVICES)
def test_the_sink_and_the_first_tokens(device, tmp_path):
    """Position 0 sees itself and its head's sink alone: with scores of 0 and sinks of log 1 and log 3, half and a
    quarter of its normed value."""
    cfg = design([(chunked(2, 2, 16, 16, 20, scale=1e-9), None)], width=32, vocab=40, mult=1.0)
    sink = torch.tensor([0.0, float(np.log(3.0))])
    eng = one_layer(tmp_path, cfg, device, lambda t: t.update({"l0.mix.sink": sink}))
    res = []
    eng.feed_step([(1, [3], [0])], residuals=res)
    w = {k: v.double() for k, v in oracle.read_checkpoint(str(tmp_path)).items()}
    x = w["embed"][[3]]
    v = oracle.rms((oracle.norm(x, w["l0.norm1"], 1e-4) @ w["l0.mix.v"].T).reshape(2, 16), 1e-4)
    o = (v * torch.tensor([[0.5], [0.25]], dtype=torch.float64)).reshape(1, 32) @ w["l0.mix.o"].T
    torch.testing.assert_close(res[0][:1].double().cpu(), x + o, rtol=1e-4, atol=1e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_equal_maps_leave_a_multiple(device, tmp_path):
    """Differential attention whose two maps are alike: (1 - lambda) times the one map, whose norm and sign remain."""
    cfg = design([(twice(2, 1, 16, 16, 16, 50.0, 0.25), None)], width=32, vocab=40)

    def alike(t):
        for k, n in (("q", 2), ("k", 1)):
            w = t[f"l0.mix.{k}"].view(n, 2, 16, 32)
            w[:, 1] = w[:, 0]
        for k, v in (("lq1", 0.5), ("lk1", 0.25), ("lq2", 0.0), ("lk2", 0.0)):  # lambda = e^2 - 1 + 0.25 > 1
            t["l0.mix." + k] = torch.full((16,), v).to(torch.bfloat16)
    eng = one_layer(tmp_path, cfg, device, alike)
    ids = torch.randint(0, 40, (40,), generator=torch.Generator().manual_seed(4)).tolist()
    tw = oracle.read_checkpoint(str(tmp_path))
    w = {k[len("l0.mix."):]: v.double() for k, v in tw.items() if k.startswith("l0.mix.")}
    assert abs(float(oracle.differential_lambda(w, 0.25)) - (float(np.exp(2.0)) - 0.75)) < 1e-12
    close(feed(eng, 1, ids, [30] + [1] * 10), oracle.forward(cfg, tw, ids), "float32")


def greedy_is_right(folder, name, prompt, out, dtype):
    lg = expect(folder, name, prompt + out[:-1])[len(prompt) - 1:]
    slack = (1e-3 if dtype == "float32" else 1.0) * float(lg.std())
    gap = torch.stack([lg[i].max() - lg[i, t] for i, t in enumerate(out)])
    assert gap.max() <= slack and gap.mean() <= 0.15 * slack, gap


@pytest.mark.parametrize("device,dtype", KINDS)
@pytest.mark.parametrize("mode", ["serial", "pipelined", "tight"])
def test_greedy_generation(folder, device, dtype, mode):
    """Through submit / scheduler / sampler, with hipGraphs on the GPU; "tight" preempts (few pages), so a
    sequence gives its slot back and starts again."""
    name = "varied"
    kw = {"tight": dict(num_kv_blocks=14), "pipelined": dict(async_steps=True, num_kv_blocks=64)}.get(mode, dict(num_kv_blocks=64))
    eng = engine(folder, name, device, dtype, use_graphs=True, prefix_caching=True, token_buckets=[4, 16, 64],
                 max_num_batched_tokens=64, max_prefill_tokens=48, **kw)
    prompts = [tokens(name, n, 70 + n) for n in (5, 61, 34, 90, 1, 17)]
    outs = eng.generate(prompts, temperature=0.0, max_tokens=12, ignore_eos=True)
    for p, o in zip(prompts, outs):
        assert len(o.token_ids) == 12
        greedy_is_right(folder, name, p, o.token_ids, dtype)
    again = eng.generate([prompts[3]], temperature=0.0, max_tokens=12, ignore_eos=True)[0]
    assert not again.cached_prompt_tokens  # states are not cached with prefixes
    greedy_is_right(folder, name, prompts[3], again.token_ids, dtype)
    assert eng.sched.num_free_states == 4


@pytest.mark.parametrize("device,dtype", KINDS)
def test_cached_prefixes(folder, device, dtype):
    """A model without recurrent layers takes prefixes from the cache, normed values included."""
    name = "attention_only"
    eng = engine(folder, name, device, dtype, prefix_caching=True, num_kv_blocks=64, max_num_batched_tokens=64, token_buckets=[4, 64])
    p = tokens(name, 90, 5)
    for want in (0, 80):
        o = eng.generate([p], temperature=0.0, max_tokens=12, ignore_eos=True)[0]
        assert (o.cached_prompt_tokens or 0) == want
        greedy_is_right(folder, name, p, o.token_ids, dtype)


@pytest.mark.gpu
def test_bucket_graphs_replay_exactly(gpu, folder):
    """A captured step replayed with other work between gives the eager step's tokens every time."""
    name = "varied"
    ids = [tokens(name, 40, 90 + i) for i in range(3)]
    want = engine(folder, name, gpu, "bfloat16", num_kv_blocks=64).generate(ids, temperature=0.0, max_tokens=20, ignore_eos=True)
    eng = engine(folder, name, gpu, "bfloat16", use_graphs=True, num_kv_blocks=64)
    for _ in range(3):
        got = eng.generate(ids, temperature=0.0, max_tokens=20, ignore_eos=True)
        torch.randn(1 << 20, device=gpu).sum().item()
        assert [o.token_ids for o in got] == [o.token_ids for o in want]
    assert eng.stats["graph_replays"] > 0


@pytest.mark.parametrize("device", DEVICES)
def test_sampling_and_embedding_requests(folder, device):
    name = "memory_first"
    eng = engine(folder, name, device, "float32", num_kv_blocks=64)
    p = tokens(name, 20)
    a = eng.generate([p] * 3, temperature=0.9, max_tokens=8, ignore_eos=True, seed=5, top_k=20, top_p=0.9)
    assert a[0].token_ids == a[1].token_ids == a[2].token_ids and max(a[0].token_ids) < 257
    e = eng.embed([p, p[:7]], pooling="mean")
    tw, lay = oracle.read_checkpoint(folder(name)), []
    oracle.forward(DESIGNS[name], tw, p, layers=lay)
    hn = oracle.norm(lay[-1], tw["final.norm"].double(), 1e-4)
    np.testing.assert_allclose(e, np.stack([hn.mean(0).numpy(), hn[:7].mean(0).numpy()]), rtol=1e-3, atol=1e-4)


def test_presets_and_parameter_counts():
    from pilottai_amd.models import registry
    from pilottai_amd.models.salipel import PRESETS, SalipelConfig

    for d in DESIGNS.values():
        assert SalipelConfig.from_dict(d).num_params() == sum(t.numel() for t in weights(d).values())
    for name in PRESETS:
        assert registry.get_config(name) is PRESETS[name]


def test_configuration_errors(folder, tmp_path):
    from pilottai_amd.models import registry
    from pilottai_amd.models.salipel import SalipelConfig

    base = DESIGNS["varied"]
    assert registry.get_config(folder("varied")).vocab_size == 101

    def changed(layer, **kw):
        d = copy.deepcopy(base)
        for k, v in kw.items():
            at = d["layers"][layer]
            *path, last = k.split("__")
            for s in path:
                at = at[s]
            at[last] = v
        return d
    for bad in (changed(0, type="other"), changed(1, mlp__kind="other"), changed(0, mixer__left__kv_heads=4), changed(0, mixer__left__vdim=20),
                changed(2, mixer__rot={"base": 10.0, "dims": 48}), changed(1, mixer__kv_heads=2), changed(0, mlp__router__top=7),
                changed(1, mixer__vdim=600), changed(2, mixer__scale=0.0)):
        with pytest.raises(ValueError):
            SalipelConfig.from_dict(bad)
    (tmp_path / "config.json").write_text(json.dumps(dict(base, width=80)))
    from safetensors.torch import save_file
    save_file(weights(base), str(tmp_path / "model.safetensors"))
    with pytest.raises(ValueError, match="shape"):
        engine(lambda _: str(tmp_path), "x", "cpu", "float32")


def test_requests_that_do_not_fit_are_refused(folder):
    eng = engine(folder, "memory_first", "cpu", "float32", num_kv_blocks=4)
    with pytest.raises(RuntimeError, match="pool"):
        eng.feed_step([(1, [3] * 40, []), (2, [3] * 40, [])])
    assert eng.sched.num_free_blocks == 4 and eng.sched.num_free_states == 4  # nothing was taken
    eng.feed_step([(i, [3], []) for i in range(4)])
    assert eng.sched.num_free_states == 0


def test_engine_registry_takes_a_folder(folder):
    """The process-wide registry that serving and agents use."""
    from pilottai_amd.engine import registry

    name = "parallel_only"
    eng = registry.get_engine(folder(name), max_model_len=128, max_num_batched_tokens=64, max_num_seqs=4)
    try:
        assert registry.get_engine(folder(name)) is eng
        p = tokens(name, 9)
        greedy_is_right(folder, name, p, eng.generate([p], temperature=0.0, max_tokens=5, ignore_eos=True)[0].token_ids, "bfloat16")
    finally:
        registry.shutdown_engines()


@pytest.mark.parametrize("device,dtype", KINDS)
def test_trace_run(folder, tmp_path, device, dtype):
    name = "varied"
    a, b = tokens(name, 30, 5), tokens(name, 12, 6)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:20], "want": [0, 19]}, {"id": "b", "tokens": b[:5], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[5:6], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[6:], "want": [5]}, {"id": "a", "tokens": a[20:], "want": [3]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "c", "tokens": b, "want": [11]}], "end": ["a", "c"]}]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder(name), "--dtype", dtype, "--out", str(tmp_path),
                        "--max-tokens", "128", "--device", device], input="\n".join(map(json.dumps, steps)) + "\n",
                       capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == [f"done {i}" for i in range(4)]
    assert not (tmp_path / "1.f32").exists()
    V = DESIGNS[name]["vocab"]
    get = lambda i: torch.from_numpy(np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(-1, V).copy())  # noqa: E731
    wa, wb = expect(folder, name, a), expect(folder, name, b)
    close(get(0), wa[[0, 19]], dtype)
    close(get(2), torch.stack([wb[11], wa[23]]), dtype)
    close(get(3), wb[11:], dtype)
