"""The Mudepel model in the engine against the plain implementation of tests/mudepel_oracle.py: whole
prompts, portions, batches, reused pages and state slots, window and block edges, long decoding and
generation, on the CPU (reference operations, fp32) and on the GPU (the kernels, fp32 and bf16)."""
import copy
import json
import os
import subprocess

import numpy as np
import pytest
import torch

import mudepel_oracle as oracle

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DEVICES = ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)]
KINDS = [("cpu", "float32"), pytest.param("cuda:0", "float32", marks=pytest.mark.gpu),
         pytest.param("cuda:0", "bfloat16", marks=pytest.mark.gpu)]


def att(heads, kv, dim, vdim, window=0, pool=0, rot=None, base=300.0, scaling=None, scale=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale or 1.3 / dim ** 0.5,
         "rot": {"base": base, "dims": rot or dim}}
    if scaling:
        m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if window:
        m["mask"] = dict({"size": window}, **({"pool": pool} if pool else {}))
    return "attention", m


def ssm(heads, vdim, state, groups, conv, norm_groups):
    return "mamba2", {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, count=0, keep=0, shared=0):
    r = {"experts": experts, "top": top}
    if count:
        r["groups"] = {"count": count, "keep": keep}
    return dict({"kind": "moe", "router": r, "expert": {"ff": ff}}, **({"shared": {"ff": shared}} if shared else {}))


def design(layers, width=72, vocab=101, streams=3, loop=None, eps=1e-4, cap=9.0):
    c = {"architecture": "Mudepel", "vocab": vocab, "width": width, "streams": streams, "norm": {"eps": eps},
         "layers": [{"type": m[0], "mixer": m[1], "mlp": p} for m, p in layers]}
    c.update({"loop": loop} if loop else {}, **({"logit_softcap": cap} if cap else {}))
    return c


DESIGNS = {
    # unequal layers: shared and own KV heads, blocks inside, at and across pages, a loop over unequal layers
    "varied": design([(att(6, 2, 40, 24, 19, 5, rot=32, scaling=(2.5, 60.0, 4.0, 1.0)), dense(56)),
                      (ssm(4, 20, 24, 2, 4, 2), moe(6, 2, 40, 3, 2, 48)),
                      (att(3, 1, 36, 36, 33, 20, rot=20), moe(5, 1, 24)),
                      (ssm(3, 16, 40, 1, 2, 1), None)], loop={"start": 1, "stop": 3, "times": 3}),
    # a recurrent layer first, blocks of a page, no rotation scaling, one stream, no cap
    "state_first": design([(ssm(6, 32, 32, 3, 6, 6), dense(100)), (att(8, 2, 64, 64, 32, 16), moe(8, 3, 64, 4, 1 + 1, 150))],
                          width=128, vocab=257, streams=1, cap=0.0, loop={"start": 1, "stop": 2, "times": 2}),
    # no recurrent layer: prefixes may be cached; no window, a window without blocks, blocks longer than the window
    "attention_only": design([(att(4, 4, 24, 40), moe(4, 2, 32, 2, 1)), (att(2, 1, 20, 10, 17), dense(33)),
                              (att(5, 5, 96, 96, 7, 24, scaling=(4.0, 32.0, 8.0, 0.5)), moe(9, 4, 20, 3, 2, 20))],
                             width=50, vocab=64, streams=2),
    # no attention layer
    "state_only": design([(ssm(5, 24, 48, 5, 3, 1), moe(7, 1, 36)), (ssm(2, 48, 16, 1, 8, 4), None)], width=64, streams=4),
    # every pair of equal things unequal, wide heads, a wide group
    "wide": design([(att(18, 1, 8, 8, 40, 3, rot=4), None), (att(3, 3, 130, 70, 25, 13, rot=130), dense(40)),
                    (ssm(8, 40, 130, 2, 5, 5), moe(12, 5, 70, 2, 1, 40))], width=96, vocab=130, streams=5, cap=30.0),
}


def weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    d, V, S = cfg["width"], cfg["vocab"], cfg["streams"]
    t = {}

    def lin(name, n, k, gain=1.0):
        t[name] = (torch.randn(n, k, generator=g) * gain / k ** 0.5).to(torch.bfloat16)

    def around(name, shape, mean, dev):
        t[name] = (mean + dev * torch.randn(shape, generator=g)).to(torch.bfloat16)

    def ff(p, f, gain=1.0):
        for k, s in (("gate", (f, d, 1.5)), ("up", (f, d, 1.5)), ("down", (d, f, gain))):
            lin(p + k, *s)

    t["embed"] = torch.randn(V, d, generator=g).to(torch.bfloat16)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        for q in (1, 2) if L["mlp"] else (1,):
            around(f"{p}norm{q}", d, 0.0, 0.2)
            around(f"{p}hc{q}.in", S, 1.0 / S, 0.15)
            around(f"{p}hc{q}.out", S, 0.6, 0.2)
            t[f"{p}hc{q}.mix"] = (0.9 * torch.eye(S) + 0.15 / S * torch.randn(S, S, generator=g)).to(torch.bfloat16)
        if L["type"] == "attention":
            for k, n, j in (("q", m["heads"] * m["dim"], d), ("k", m["kv_heads"] * m["dim"], d),
                            ("v", m["kv_heads"] * m["vdim"], d), ("o", d, m["heads"] * m["vdim"])):
                lin(p + "mix." + k, n, j)
                around(f"{p}mix.{k}.b", n, 0.0, 0.3)
        else:
            inner, bc, H = m["heads"] * m["vdim"], 2 * m["groups"] * m["state"], m["heads"]
            lin(p + "mix.in", 2 * inner + bc + H, d, 1.2)
            around(p + "mix.conv", (inner + bc, m["conv"]), 0.0, 0.5)
            around(p + "mix.conv.b", inner + bc, 0.0, 0.2)
            around(p + "mix.dt_bias", H, -2.0, 0.7)
            t[p + "mix.A_log"] = torch.log(torch.linspace(0.05, 4.0, H)).to(torch.bfloat16)  # long and short memories
            around(p + "mix.D", H, 0.7, 0.3)
            around(p + "mix.norm", inner, 1.0, 0.2)
            lin(p + "mix.o", d, inner)
        f = L["mlp"]
        if f and f["kind"] == "dense":
            ff(p + "mlp.", f["ff"])
        elif f:
            lin(p + "mlp.router", f["router"]["experts"], d, 2.0)
            for e in range(f["router"]["experts"]):
                ff(f"{p}mlp.e{e}.", f["expert"]["ff"], 0.25)  # (a close call in bf16 swaps an expert: of limited weight)
            if f.get("shared"):
                ff(p + "mlp.shared.", f["shared"]["ff"])
    around("final.norm", d, 0.0, 0.2)
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
@pytest.mark.parametrize("name", ["state_first", "attention_only", "state_only", "wide"])
def test_portions_of_every_design(folder, name, device, dtype):
    eng = engine(folder, name, device, dtype)
    ids = tokens(name, 150)
    close(feed(eng, 1, ids, [7, 2, 1, 1, 30, 3, 66, 2, 8] + [1] * 30), expect(folder, name, ids), dtype)


@pytest.mark.parametrize("device,dtype", KINDS)
@pytest.mark.parametrize("name", ["varied", "state_first"])
def test_residual_after_every_run(folder, name, device, dtype):
    eng = engine(folder, name, device, dtype)
    ids = tokens(name, 29)
    want, got = [], []
    oracle.forward(DESIGNS[name], oracle.read_checkpoint(folder(name)), ids, layers=want)
    eng.feed_step([(1, ids, [0])], residuals=got)
    assert len(got) == len(want) == len(oracle.runs(DESIGNS[name]))
    for j, (g, w) in enumerate(zip(got, want)):
        close(g[:len(ids)], w, dtype, f"run {j}")


@pytest.mark.parametrize("device,dtype", KINDS)
@pytest.mark.parametrize("name", ["varied", "state_only"])
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
    name = "state_first"
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
    name = "state_only"
    eng = engine(folder, name, device, "float32", max_num_seqs=1, num_kv_blocks=16)
    for seed, cuts in ((1, [70]), (2, [1] * 20), (3, [2] * 10), (4, [12])):
        ids = tokens(name, sum(cuts), seed)
        close(feed(eng, seed, ids, cuts), expect(folder, name, ids), "float32", f"seed {seed}")
        eng.release_fed(seed)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("W,P", [(21, 6), (16, 16), (5, 9), (40, 1), (33, 40), (12, 0)])
def test_what_a_position_sees(device, tmp_path, W, P):
    """One attention layer: another token changes the last position's logits exactly if it lies in the window
    or in a block that is wholly before it, in whole prompts, in portions and in decoding."""
    from safetensors.torch import save_file

    cfg = design([(att(2, 1, 16, 16, W, P), None)], width=32, vocab=40, streams=2)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(weights(cfg), str(tmp_path / "model.safetensors"))
    eng = engine(lambda _: str(tmp_path), "", device, "float32", max_num_batched_tokens=128)
    n = 90
    ids = torch.randint(0, 40, (n,), generator=torch.Generator().manual_seed(W)).tolist()
    last, seen_blocks = n - 1, max(0, n - W) // P if P else 0
    places = {last - W + 1: True, last - W: last - W < seen_blocks * P, 0: seen_blocks > 0, 1: seen_blocks * P > 1}
    if P:
        places.update({seen_blocks * P - 1: True, seen_blocks * P: seen_blocks * P > last - W})
    base = oracle.forward(cfg, oracle.read_checkpoint(str(tmp_path)), ids)[-1]
    for j, seen in places.items():
        if not 0 <= j < last:
            continue
        other = list(ids)
        other[j] = (other[j] + 1) % 40
        for cuts in ([n], [64] + [1] * 26, [2] * 45, [30, 37, 23]):
            got = feed(eng, 2, other, cuts)[-1].double().cpu()
            eng.release_fed(2)
            assert ((got - base).abs().max() > 1e-4) == seen, (j, seen, cuts[:3], float((got - base).abs().max()))


@pytest.mark.parametrize("device", DEVICES)
def test_the_sink_and_the_first_tokens(device, tmp_path):
    """Position 0 sees itself and the sink alone: with scores near 0 it gets half its value."""
    from safetensors.torch import save_file

    cfg = design([(att(2, 2, 16, 16, 20, 4, scale=1e-6), None)], width=32, vocab=40, streams=1, cap=0.0)
    tw = weights(cfg)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(tw, str(tmp_path / "model.safetensors"))
    eng = engine(lambda _: str(tmp_path), "", device, "float32")
    res = []
    eng.feed_step([(1, [3, 5, 7], [0])], residuals=res)
    w = {k: v.double() for k, v in tw.items()}
    x = w["embed"][[3, 5, 7]]
    v = oracle.norm(w["l0.hc1.in"] * x, w["l0.norm1"], 1e-4) @ w["l0.mix.v"].T + w["l0.mix.v.b"]
    o = v.cumsum(0) / torch.tensor([[2.0], [3.0], [4.0]], dtype=torch.float64) @ w["l0.mix.o"].T + w["l0.mix.o.b"]
    torch.testing.assert_close(res[0][:3].double().cpu(), w["l0.hc1.mix"] * x + w["l0.hc1.out"] * o, rtol=1e-4, atol=1e-4)


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
def test_cached_prefixes_keep_their_pooled_blocks(folder, device, dtype):
    """A model without recurrent layers takes prefixes from the cache, pooled rows included."""
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
    name = "state_first"
    eng = engine(folder, name, device, "float32", num_kv_blocks=64)
    p = tokens(name, 20)
    a = eng.generate([p] * 3, temperature=0.9, max_tokens=8, ignore_eos=True, seed=5, top_k=20, top_p=0.9)
    assert a[0].token_ids == a[1].token_ids == a[2].token_ids and max(a[0].token_ids) < 257
    e = eng.embed([p, p[:7]], pooling="mean")
    tw, lay = oracle.read_checkpoint(folder(name)), []
    oracle.forward(DESIGNS[name], tw, p, layers=lay)
    hn = oracle.norm(lay[-1], tw["final.norm"].double(), 1e-4)
    np.testing.assert_allclose(e, np.stack([hn.mean(0).numpy(), hn[:7].mean(0).numpy()]), rtol=1e-3, atol=1e-4)


def test_runs_and_presets():
    from pilottai_amd.models import registry
    from pilottai_amd.models.mudepel import PRESETS, MudepelConfig

    assert MudepelConfig.from_dict(DESIGNS["varied"]).runs() == [0, 1, 2, 1, 2, 1, 2, 3]
    for d in DESIGNS.values():
        c = MudepelConfig.from_dict(d)
        assert c.runs() == oracle.runs(d)
        assert c.num_params() == sum(t.numel() for t in weights(d).values())
    for name in PRESETS:
        assert registry.get_config(name) is PRESETS[name]


def test_configuration_errors(folder, tmp_path):
    from pilottai_amd.models import registry
    from pilottai_amd.models.mudepel import MudepelConfig

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
    for bad in (changed(0, type="other"), changed(0, mlp__kind="other"), changed(0, mixer__kv_heads=4),
                changed(0, mixer__rot={"base": 10.0, "dims": 48}), changed(1, mixer__groups=3),
                changed(1, mlp__router__groups={"count": 4, "keep": 1}), changed(1, mlp__router__groups={"count": 3, "keep": 4}),
                changed(1, mlp__router__top=5), dict(base, loop={"start": 1, "stop": 9, "times": 2})):
        with pytest.raises(ValueError):
            MudepelConfig.from_dict(bad)
    (tmp_path / "config.json").write_text(json.dumps(dict(base, width=80)))
    from safetensors.torch import save_file
    save_file(weights(base), str(tmp_path / "model.safetensors"))
    with pytest.raises(ValueError, match="shape"):
        engine(lambda _: str(tmp_path), "x", "cpu", "float32")


def test_requests_that_do_not_fit_are_refused(folder):
    eng = engine(folder, "state_first", "cpu", "float32", num_kv_blocks=4)
    with pytest.raises(RuntimeError, match="pool"):
        eng.feed_step([(1, [3] * 40, []), (2, [3] * 40, [])])
    assert eng.sched.num_free_blocks == 4 and eng.sched.num_free_states == 4  # nothing was taken
    with pytest.raises(RuntimeError, match="slots"):
        eng.feed_step([(i, [3], []) for i in range(5)])
    eng.feed_step([(i, [3], []) for i in range(4)])
    assert eng.sched.num_free_states == 0
    eng.release_fed(2)
    eng.feed_step([(9, [3], [0])])
    with pytest.raises(KeyError):
        eng.release_fed(2)


def test_engine_registry_takes_a_folder(folder):
    """The process-wide registry that serving and agents use."""
    from pilottai_amd.engine import registry

    eng = registry.get_engine(folder("state_only"), max_model_len=128, max_num_batched_tokens=64, max_num_seqs=4)
    try:
        assert registry.get_engine(folder("state_only")) is eng
        p = tokens("state_only", 9)
        greedy_is_right(folder, "state_only", p, eng.generate([p], temperature=0.0, max_tokens=5, ignore_eos=True)[0].token_ids, "bfloat16")
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
