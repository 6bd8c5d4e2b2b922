"""GPU tests of the Foderax serving path against the plain oracle (oracle/foderax.py): each mechanism's kernel alone, then the model through the registry,
the slot cache and the ragged-batch scheduler -- whole prompts, token-by-token decoding, portions, unequal batches, reused slots, far keys, long decoding,
odd sizes, greedy generation, the trace replay program.  fp32 mode is held to fp32 rounding; bf16 mode to a few bf16 roundings of the logits' scale."""

import copy
import json
import os
import subprocess
import sys

import pytest
import torch

from oracle import foderax as O
from tests import foderax_util as U

pytestmark = pytest.mark.gpu
_oracle_cache = {}
DEV = "cuda"
F32, F64, BF16, I32 = torch.float32, torch.float64, torch.bfloat16, torch.int32
TOL = {"float32": 3e-5, "bfloat16": 8e-2}


def dev_i32(x):
    return torch.tensor(x, dtype=I32).to(DEV)


def row_err(got, want):
    """The worst row's rms of the difference (mean removed) over the rms of the wanted rows."""
    got, want = got.detach().double().cpu(), want.detach().double().cpu()
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    return (d.pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()).max().item()


def tokens(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def all_experts(cfg):
    """The same configuration with every group kept and every expert chosen.  A top-k choice is no continuous function: where two router scores nearly tie, bf16
    rounding upstream may pick the other expert, which says nothing about the kernels -- so the bf16 runs of whole models route every token to every expert
    (dispatch, weights and epilogue are all still there), and the choice itself is tested in fp32 and on the router kernel alone."""
    cfg = copy.deepcopy(cfg)
    for layer in cfg["layers"]:
        if layer.get("mlp"):
            r = layer["mlp"]["router"]
            r["top"], r["groups"]["keep"] = r["experts"], r["groups"]["count"]
    return cfg


def clear_tokens(cfg, w, n, seed, margin=1e-3):
    """Random tokens on which no router makes a close call at fp32 rounding: the seed is stepped until every token's gap exceeds ``margin``."""
    for k in range(60):
        toks = tokens(n, cfg["vocab"], seed + 1000 * k)
        gaps = []
        _oracle_cache[(id(w), str(cfg["layers"]), tuple(toks), False)] = O.forward(cfg, w, toks, F64, gaps=gaps)
        if not gaps or min(float(g_.min()) for g_ in gaps) > margin:
            return toks
    raise AssertionError("no token sequence without a close router call found")


@pytest.fixture(scope="module")
def checkpoint(tmp_path_factory):
    cfg = U.make_config(U.default_layers())
    w = U.make_weights(cfg, 11)
    return U.save(str(tmp_path_factory.mktemp("foderax")), cfg, w), cfg, w


@pytest.fixture(scope="module")
def models(checkpoint, tmp_path_factory):
    """dtype -> (model, its configuration, weights): the bf16 model chooses every expert (``all_experts``), on the same weights."""
    from llm_quest_amd import registry

    folder, cfg, w = checkpoint
    every = all_experts(cfg)
    folder16 = U.save(str(tmp_path_factory.mktemp("foderax16")), every, w)
    return {"float32": (registry.load_model(folder, "float32", DEV), cfg, w), "bfloat16": (registry.load_model(folder16, "bfloat16", DEV), every, w)}


def oracle(cfg, w, toks, layers=False):
    key = (id(w), str(cfg["layers"]), tuple(toks), layers)
    if key not in _oracle_cache:
        _oracle_cache[key] = O.forward(cfg, w, toks, F64, return_layers=layers)
    return _oracle_cache[key]


def batch_of(model, **kw):
    from llm_quest_amd.generate import RaggedBatch

    return RaggedBatch(model, **kw)


# ------------------------------------------------------------------------------------------------------------------- the model through the scheduler
@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
def test_whole_prompt_every_layer(models, dt):
    model, cfg, w = models[dt]
    toks = clear_tokens(cfg, w, 70, 1)
    want, layers = oracle(cfg, w, toks, layers=True)
    got, got_layers = batch_of(model).step([("a", toks)], [list(range(len(toks)))], return_layers=True)
    assert len(got_layers) == len(layers)
    for i, l in enumerate(got_layers):
        assert row_err(l, layers[i]) < TOL[dt], f"stream after layer {i}"
    assert row_err(got, want) < TOL[dt]


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
def test_token_by_token_from_the_first_token(models, dt):
    """Every token alone: the first one sees itself and the sinks, the recurrences start at zero; the one-token form of every kernel from the first token on."""
    model, cfg, w = models[dt]
    toks = clear_tokens(cfg, w, 60, 2)
    b = batch_of(model)
    got = torch.cat([b.step([("a", [t])]) for t in toks])
    assert row_err(got, oracle(cfg, w, toks)) < TOL[dt]


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
def test_portions_of_several_sizes(models, dt):
    """Portions down to one and two tokens: the first is a prompt, the others go on against the cache."""
    model, cfg, w = models[dt]
    toks = clear_tokens(cfg, w, 90, 3)
    b = batch_of(model)
    got, at = [], 0
    for n in [7, 2, 2, 1, 1, 33, 1, 9, 2, 32]:
        got.append(b.step([("a", toks[at : at + n])], [list(range(n))]))
        at += n
    assert at == len(toks)
    assert row_err(torch.cat(got), oracle(cfg, w, toks)) < TOL[dt]


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
def test_unequal_batch_equals_each_request_alone(models, dt):
    model, cfg, w = models[dt]
    lens, tail = [1, 41, 17, 66], 9
    seqs = [clear_tokens(cfg, w, n + tail, 10 + i) for i, n in enumerate(lens)]
    alone = [batch_of(model).step([("x", s)], [list(range(len(s)))]) for s in seqs]
    b = batch_of(model, slots=2)  # fewer slots than sequences: the cache grows
    got = [[] for _ in seqs]
    out = b.step([(i, s[: lens[i]]) for i, s in enumerate(seqs)], [list(range(n)) for n in lens])
    at = 0
    for i, n in enumerate(lens):
        got[i].append(out[at : at + n])
        at += n
    live = list(range(len(seqs)))
    for k in range(tail):
        if k == 4:  # two requests leave early; the others go on
            for i in (0, 2):
                b.finish(i)
                live.remove(i)
        out = b.step([(i, [seqs[i][lens[i] + k]]) for i in live])
        for j, i in enumerate(live):
            got[i].append(out[j : j + 1])
    for i, s in enumerate(seqs):
        g = torch.cat(got[i])
        ref = alone[i][: g.shape[0]]  # (alone, the whole request is one prompt: in bf16 its last tokens take the prompt form of the kernels, here the one-token form)
        assert row_err(g, ref) < (1e-5 if dt == "float32" else 6e-2), f"request {i} in the batch differs from the request alone"
        assert row_err(g, oracle(cfg, w, s)[: g.shape[0]]) < TOL[dt]


def test_mixed_batch_of_prompts_portions_and_single_tokens(models):
    """One step holds a new prompt, a portion of an older one and a single token of a third; each equals the request alone."""
    model, cfg, w = models["float32"]
    seqs = [clear_tokens(cfg, w, n, 60 + n) for n in (40, 35, 30)]
    b = batch_of(model)
    got = {0: [b.step([(0, seqs[0][:25])], [list(range(25))])], 1: [], 2: []}
    cuts = [[(0, 25, 26), (1, 0, 20)], [(0, 26, 39), (1, 20, 21), (2, 0, 28)], [(1, 21, 35), (0, 39, 40), (2, 28, 30)]]
    for step in cuts:
        out = b.step([(i, seqs[i][a:e]) for i, a, e in step], [list(range(e - a)) for _, a, e in step])
        at = 0
        for i, a, e in step:
            got[i].append(out[at : at + e - a])
            at += e - a
    for i, s in enumerate(seqs):
        assert row_err(torch.cat(got[i]), oracle(cfg, w, s)) < TOL["float32"], i


def test_freed_slots_are_reused_without_leftovers(models):
    """A long sequence leaves key / value and latent rows and recurrent states behind; the next, shorter one takes its slot and must see none of them.  The
    cache starts small, so rows also grow while a sequence is alive."""
    model, cfg, w = models["float32"]
    b = batch_of(model, slots=1)
    b.cache.initial_chunk_size, b.cache.chunk_size = 4, 8
    long_, short = tokens(60, cfg["vocab"], 20), clear_tokens(cfg, w, 33, 21)
    b.step([("long", long_[:50])])
    for t in long_[50:]:
        b.step([("long", [t])])
    b.finish("long")
    got = [b.step([("short", short[:12])], [list(range(12))])] + [b.step([("short", [t])]) for t in short[12:]]
    assert b.cache.reuses >= 1 and b.cache.slots == 1
    assert row_err(torch.cat(got), oracle(cfg, w, short)) < TOL["float32"]


def test_long_decoding(models):
    """220 decoded tokens over every key so far; the recurrent states are carried all the way."""
    model, cfg, w = models["float32"]
    toks = clear_tokens(cfg, w, 225, 30, margin=2e-4)
    b = batch_of(model)
    b.step([("a", toks[:5])])
    got = torch.cat([b.step([("a", [t])]) for t in toks[5:]])
    assert row_err(got, oracle(cfg, w, toks)[5:]) < TOL["float32"]


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
def test_long_prompt_then_decoding_with_dealt_out_keys(tmp_path, dt):
    """700 keys: one-token steps deal a tile's keys to several workgroups whose partial results meet (softmax, sink and sigmoid weights)."""
    from llm_quest_amd import registry

    cfg = U.make_config([(U.latent(), None), (U.diff(), None), (U.parallel(), None), (U.diff(kv_from=1), None)])
    w = U.make_weights(cfg, 3)
    model = registry.load_model(U.save(str(tmp_path), cfg, w), dt, DEV)
    toks = tokens(704, cfg["vocab"], 4)
    want = oracle(cfg, w, toks)
    other = tokens(97, cfg["vocab"], 5)  # a shorter request beside it: most of its share of the deal is empty
    want2 = oracle(cfg, w, other)
    b = batch_of(model)
    got = b.step([("a", toks[:697]), ("b", other[:90])], [[0, 1, 350, 696], [89]])
    assert row_err(got[:4], want[[0, 1, 350, 696]]) < TOL[dt] and row_err(got[4:], want2[89:90]) < TOL[dt]
    got = torch.stack([b.step([("a", [t]), ("b", [u])]) for t, u in zip(toks[697:], other[90:])])
    assert row_err(got[:, 0], want[697:]) < TOL[dt] and row_err(got[:, 1], want2[90:]) < TOL[dt]


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
def test_other_sizes_odd_and_one(tmp_path, dt):
    """Sizes that are no multiples of 8 or of each other's: one head, one key head per query head, latents of one and of odd sizes, a rotation of two entries and of
    none, no feed-forward, one expert, one group, every group kept, a recurrence of odd width, factors of 0 and 1, no cap, an embedding scale of 1, value heads
    wider than the queries and narrower, one layer's keys read by two later ones."""
    from llm_quest_amd import registry

    layers = [(U.diff(heads=1, kv_heads=1, dim=6, vdim=5, rot_dims=2, base=3.0, diff=0.0), None),
              (U.diff(heads=5, kv_heads=1, dim=6, vdim=5, rot_dims=2, base=3.0, diff=0.9, kv_from=0), U.moe(experts=1, top=1, ff=20, count=1, keep=1)),
              (U.latent(heads=1, dim=7, vdim=13, q_rank=1, kv_rank=9, scale=1.0), U.moe(experts=4, top=4, ff=33, count=2, keep=2)),
              (U.diff(heads=2, kv_heads=1, dim=6, vdim=5, rot_dims=6, base=3.0, kv_from=0), None),
              (U.parallel(heads=1, kv_heads=1, dim=3, vdim=41, rot_dims=0, width=1, left_scale=1.0, right_scale=1.0), U.moe(experts=6, top=1, ff=7, count=3, keep=1)),
              (U.parallel(heads=7, kv_heads=7, dim=14, vdim=2, rot_dims=14, width=77, left_scale=0.0, right_scale=2.0), U.moe(experts=9, top=3, ff=12, count=9, keep=4)),
              (U.latent(heads=5, dim=33, vdim=3, q_rank=50, kv_rank=70), None)]
    layers[3][0]["mixer"]["rot"] = dict(layers[0][0]["mixer"]["rot"])
    cfg = U.make_config(layers, width=100, vocab=77, eps=1e-6, scale=1.0, softcap=0.0)
    del cfg["logit_softcap"]
    w = U.make_weights(cfg, 5)
    cfg = cfg if dt == "float32" else all_experts(cfg)
    model = registry.load_model(U.save(str(tmp_path), cfg, w), dt, DEV)
    toks = clear_tokens(cfg, w, 48, 6)
    b = batch_of(model)
    got = [b.step([("a", toks[:29])], [list(range(29))])] + [b.step([("a", toks[29:31])], [[0, 1]])] + [b.step([("a", [t])]) for t in toks[31:]]
    assert row_err(torch.cat(got), oracle(cfg, w, toks)) < TOL[dt]


def test_wide_rows_and_wide_heads(tmp_path):
    """Rows wider than 512, maps of 136 and 72 with values of 136, heads beyond what the MFMA kernel keeps in registers (values of 264), a latent of 330."""
    from llm_quest_amd import registry

    layers = [(U.diff(heads=2, kv_heads=1, dim=136, vdim=136, rot_dims=64), U.moe(ff=64)),
              (U.latent(heads=2, dim=72, vdim=72, q_rank=64, kv_rank=330), None),
              (U.parallel(heads=2, kv_heads=1, dim=200, vdim=264, rot_dims=128, width=520), U.moe(ff=16)),
              (U.diff(heads=4, kv_heads=2, dim=72, vdim=264, rot_dims=72), None)]
    cfg0 = U.make_config(layers, width=520, vocab=50)
    w = U.make_weights(cfg0, 9)
    for dt in ("float32", "bfloat16"):
        cfg = cfg0 if dt == "float32" else all_experts(cfg0)
        toks = clear_tokens(cfg, w, 40, 8)
        model = registry.load_model(U.save(str(tmp_path / dt), cfg, w), dt, DEV)
        b = batch_of(model)
        got = [b.step([("a", toks[:21])], [list(range(21))])] + [b.step([("a", [t])]) for t in toks[21:]]
        assert row_err(torch.cat(got), oracle(cfg, w, toks)) < TOL[dt]


def test_greedy_generation_through_the_entry_point(models):
    from llm_quest_amd.generate import generate_ragged

    model, cfg, w = models["float32"]
    prompts = [tokens(n, cfg["vocab"], 40 + n) for n in (4, 19, 9)]
    out = generate_ragged(model, prompts, max_gen=10)
    for p, gen in zip(prompts, out):
        assert len(gen) == 10
        seq = list(p)
        for t in gen:
            lg = O.forward(cfg, w, seq, F64)[-1]
            top = torch.topk(lg, 2)
            if int(top.indices[0]) != t:
                assert float(top.values[0] - top.values[1]) < 1e-4, "greedy token differs from the oracle's without a near tie"
                break
            seq.append(t)
    first = out[1][2]
    out2 = generate_ragged(model, prompts, max_gen=10, eos_ids=[first])
    assert out2[1] == out[1][: out[1].index(first)] and out2[0] == out[0][: len(out2[0])]


def test_trace_replay_program_end_to_end(checkpoint, tmp_path):
    """bin/trace_run as a user runs it: a folder, steps on standard input (two prompts in one batch, then one token each, one request ending early and
    its slot taken by a third), logits files out -- against the oracle."""
    folder32, cfg32, w = checkpoint
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    every = all_experts(cfg32)
    for dt, (folder, cfg) in {"float32": (folder32, cfg32), "bfloat16": (U.save(str(tmp_path / "every"), every, w), every)}.items():
        _replay(root, folder, cfg, w, dt, tmp_path / dt)


def _replay(root, folder, cfg, w, dt, out):
    import numpy as np

    a, b, c = clear_tokens(cfg, w, 31, 50), clear_tokens(cfg, w, 9, 51), clear_tokens(cfg, w, 12, 52)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:28], "want": [0, 13, 27]}, {"id": "b", "tokens": b[:8], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[28:29], "want": [0]}, {"id": "b", "tokens": b[8:9], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[29:30], "want": []}], "end": []},
             {"step": 3, "entries": [{"id": "c", "tokens": c, "want": [11]}], "end": ["c"]},
             {"step": 4, "entries": [{"id": "a", "tokens": a[30:31], "want": [0]}], "end": ["a"]}]
    wa, wb, wc = oracle(cfg, w, a), oracle(cfg, w, b), oracle(cfg, w, c)
    want = {0: torch.stack([wa[0], wa[13], wa[27]]), 1: torch.stack([wa[28], wb[8]]), 3: wc[11:12], 4: wa[30:31]}
    res = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", dt, "--out", str(out), "--max-tokens", "64"],
                         input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=100)
    assert res.returncode == 0, res.stderr[-2000:]
    assert [l for l in res.stdout.split("\n") if l.startswith("done")] == [f"done {i}" for i in range(5)]
    assert not (out / "2.f32").exists()
    for i, ref in want.items():
        got = torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, cfg["vocab"]))
        assert got.shape == ref.shape and row_err(got, ref) < TOL[dt], (dt, i)


# ------------------------------------------------------------------------------------------------------------------- mechanisms alone
@pytest.mark.parametrize("width", [72, 100, 250, 256, 520, 1000, 2048, 4100])
def test_parallel_sum_depth_average_and_norm(width):
    from llm_quest_amd import kernels_seq as S

    g = torch.Generator().manual_seed(width)
    T, parts, eps = 9, 3, 1e-5
    r = lambda *s: torch.randn(*s, generator=g)
    x, ya, yb, y2, ls1, ls2, w = r(T, width) * 3, r(T, width), r(T, width), r(T * parts, width), r(width), r(width), 1.0 + 0.3 * r(width)
    d = lambda t: t.to(DEV)
    for n_hist in (0, 1, 4):
        for ydt in (F32, BF16):
            hist, dwa = r(n_hist + 3, T, width), r(n_hist + 1)
            a, b, e = ya.to(ydt), yb.to(ydt), y2.to(ydt)
            v = x.double() + ls1.double() * (0.7 * a.double() + 1.3 * b.double()) + ls2.double() * e.double().reshape(T, parts, width).sum(1)
            xa = sum(dwa[j].double() * hist[j].double() for j in range(n_hist)) + dwa[n_hist].double() * v
            hd = d(hist)
            x_out, h, h32 = S.depth_sum(d(x), ya=d(a), ca=0.7, yb=d(b), cb=1.3, ls1=d(ls1), y2=d(e), parts=parts, ls2=d(ls2), hist=hd, n_hist=n_hist, d=d(dwa), x_out=True, norm=d(w),
                                        eps=eps, out_dtype=BF16, want32=True)
            assert torch.allclose(x_out.cpu().double(), xa, atol=1e-4) and torch.allclose(hd[n_hist].cpu().double(), v, atol=3e-5)
            keep = [j for j in range(n_hist + 3) if j != n_hist]
            assert torch.equal(hd[keep].cpu(), hist[keep])  # no other result is touched
            assert row_err(h32, O.unit_rms(xa, eps) * w.double()) < 3e-6 and torch.equal(h.cpu(), h32.cpu().to(BF16))
    # one branch, no feed-forward, no scale, a summand on a view with a pitch of its own; the norm alone, where eps decides
    wide = d(torch.cat([ya, yb], dim=1))
    hd, dwa = d(r(2, T, width)), d(torch.tensor([0.0, 1.0]))
    x_out, none, _ = S.depth_sum(d(x), ya=wide[:, width:], hist=hd, n_hist=1, d=dwa, x_out=True)
    assert none is None and torch.allclose(x_out.cpu().double(), x.double() + yb.double(), atol=3e-5)
    _, h, _ = S.depth_sum(d(x * 1e-3), norm=d(w), eps=eps, out_dtype=F32)
    assert row_err(h, O.unit_rms(x.double() * 1e-3, eps) * w.double()) < 3e-6


@pytest.mark.parametrize("H,D", [(3, 24), (1, 1), (5, 7), (2, 64), (4, 128), (2, 136), (1, 264), (3, 66)])
def test_difference_of_two_maps_to_unit_rms(H, D):
    from llm_quest_amd import kernels_seq as S

    g = torch.Generator().manual_seed(D)
    T, eps, lam, c = 11, 1e-5, 0.8, 0.4
    a1, gate = torch.randn(T, H * D, generator=g), torch.randn(T, H * D + 5, generator=g)
    a2 = a1 / lam + torch.cat([torch.full((4, H * D), 1e-3), torch.ones(T - 4, H * D)]) * torch.randn(T, H * D, generator=g)  # rows where the maps all but cancel
    o = O.unit_rms((a1.double() - lam * a2.double()).reshape(T, H, D), eps).reshape(T, H * D) * c
    for gdt in (F32, BF16):
        gd = gate.to(gdt).to(DEV)[:, 5:]
        want = o * torch.sigmoid(gd.cpu().double())
        got = S.diff_join(a1.to(DEV), a2.to(DEV), H, D, lam, eps, c, gd, F32)
        assert torch.allclose(got.cpu().double(), want, atol=3e-4 if D > 1 else 2e-3), (H, D)
        assert row_err(got[4:], want[4:]) < 3e-6
        assert row_err(S.diff_join(a1.to(DEV), a2.to(DEV), H, D, lam, eps, c, gd, BF16)[4:], want[4:]) < 6e-3
    assert row_err(S.diff_join(a1.to(DEV), a2.to(DEV), H, D, lam, eps, c, None, F32)[4:], o[4:]) < 3e-6


def _kv_case(n, past, H, G, d, dv, dt, seed, boost=None, maps=1):
    """Queries [n_new, H * maps * d] and a cache [G x maps x d | G x dv] of n rows behind five foreign rows.  ``boost`` = (query position, key position, map): that
    query and key are made parallel and long, so that the key dominates the row."""
    g = torch.Generator().manual_seed(seed)
    q, k, v = torch.randn(n, H, maps, d, generator=g), torch.randn(n, G, maps, d, generator=g), torch.randn(n, G, dv, generator=g)
    if boost:
        qi, kj, mp = boost
        q[qi, :, mp] = 4.0 * k[kj, :, mp].repeat_interleave(H // G, dim=0)
        k[kj, :, mp] = 3.0 * k[kj, :, mp]
    kv_dt = BF16 if dt == "bfloat16" else F32
    k, v = k.to(kv_dt), v.to(kv_dt)
    cache = torch.full((5 + n + 3, G * (maps * d + dv)), 7.0, dtype=kv_dt, device=DEV)
    cache[5 : 5 + n] = torch.cat([k.reshape(n, -1), v.reshape(n, -1)], dim=1).to(DEV)
    desc = (dev_i32([0]), dev_i32([n - past]), dev_i32([past]), dev_i32([5]), dev_i32([5]), dev_i32([5]))
    return q.double(), k.double(), v.double(), q[past:].reshape(n - past, -1).contiguous().to(DEV), cache, desc


CASES = [(70, 0), (200, 0), (127, 37), (701, 700), (1500, 1499), (132, 129), (15, 10), (64, 0), (65, 64), (1, 0), (2, 0)]


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["sink", "sigmoid"])
def test_attention_with_a_sink_or_without_a_softmax(dt, kind):
    """Prompts, portions and one-token steps (dealt out over long caches); then single keys made dominant, near and hundreds of positions away, at the edges
    of the kernels' 64-key steps; a sink that takes nearly everything and one that takes nothing; biases that open and close every key."""
    from llm_quest_amd import kernels_seq as S

    tol = 2e-5 if dt == "float32" else 2e-2
    H, G, d, dv, scale = 4, 2, 24, 40, 0.3
    boosts = [(70, 0, (69, 0, 0)), (200, 0, (199, 63, 0)), (200, 0, (130, 64, 0)), (701, 700, (700, 0, 0)), (701, 700, (700, 255, 0)), (701, 700, (700, 700, 0)), (132, 129, (130, 128, 0))]
    for n, past, boost in [(n, p, None) for n, p in CASES] + boosts:
        for extra in ([-9.0, 0.0, 1.5, 6.0], [0.3, 0.3, 0.3, 0.3]):
            q, k, v, qd, cache, desc = _kv_case(n, past, H, G, d, dv, dt, n + past, boost)
            e = torch.tensor(extra)
            out = torch.empty(n - past, H * dv, dtype=cache.dtype, device=DEV)
            S.latent_attn(qd, cache, None, cache[:, G * d :], out, H, 2, d, 0, dv, d, d, dv, dv, desc, n - past, scale, max_keys=n, kv_rep=H // G,
                          **({"sink": e.to(DEV)} if kind == "sink" else {"sig_bias": e.to(DEV)}))
            for h in range(H):
                one = O.softmax_map if kind == "sink" else O.sigmoid_map
                want = one(q[:, h, 0], k[:, h // 2, 0], v[:, h // 2], scale, e[h].double())[past:]
                got = out[:, h * dv : (h + 1) * dv].double().cpu()
                ref = max(float(want.abs().max()), 1e-6)
                assert float((got - want).abs().max()) / ref < tol, (n, past, boost, h, extra)


@pytest.mark.parametrize("D1,D2,DV", [(128, 0, 128), (128, 64, 128), (256, 0, 256), (256, 64, 256), (200, 0, 40), (64, 0, 200), (320, 0, 16), (32, 8, 72), (136, 40, 256)])
def test_attention_over_every_key_at_every_width(D1, D2, DV):
    """bf16 keys of one and of two parts (the second shared by the heads), every width class of the kernel, prompts, portions and dealt-out one-token steps, a
    sink, fp32 and bf16 output; three sequences of unequal lengths in one launch against each alone."""
    from llm_quest_amd import kernels_seq as S

    g = torch.Generator().manual_seed(D1 + DV)
    H, scale = 3, (D1 + D2) ** -0.5
    sink = torch.tensor([0.5, -2.0, 2.0])
    for new, past in (([70, 5, 129], [0, 0, 0]), ([1, 1, 1], [600, 3, 64]), ([2, 33, 1], [90, 31, 63])):
        q = torch.randn(sum(new), H * (D1 + D2), generator=g) * 2
        n = [a + b for a, b in zip(new, past)]
        cap = max(n) + 4
        k1, k2, v = (torch.randn(3 * cap, w, generator=g).to(BF16) for w in (H * D1, max(D2, 8), H * DV))
        q_row0, row0 = [0, new[0], new[0] + new[1]], [cap * i for i in range(3)]
        desc = tuple(dev_i32(t) for t in (q_row0, new, past, row0, row0, row0))
        for o_dt in (F32, BF16):
            out = torch.zeros(sum(new), H * DV, dtype=o_dt, device=DEV)
            k1d, k2d, vd = k1.to(DEV), k2.to(DEV), v.to(DEV)
            S.latent_attn(q.to(DEV), k1d, k2d[:, :D2] if D2 else None, vd, out, H, 1, D1, D2, DV, D1 + D2, D1, DV, DV, desc, max(new), scale, max_keys=max(n), sink=sink.to(DEV))
            for s in range(3):
                rows = slice(row0[s], row0[s] + n[s])
                for h in range(H):
                    kk = torch.cat([k1[rows, h * D1 : (h + 1) * D1], k2[rows, :D2]], dim=1).double()
                    qq = torch.zeros(n[s], D1 + D2, dtype=F64)
                    qq[past[s] :] = q[q_row0[s] : q_row0[s] + new[s], h * (D1 + D2) : (h + 1) * (D1 + D2)].double()
                    want = O.softmax_map(qq, kk, v[rows, h * DV : (h + 1) * DV].double(), scale, sink[h].double())[past[s] :]
                    got = out[q_row0[s] : q_row0[s] + new[s], h * DV : (h + 1) * DV].double().cpu()
                    assert float((got - want).abs().max()) < 3e-2 * float(want.abs().max()), (new, past, s, h, o_dt)


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,G,d,dv", [(4, 2, 16, 24), (3, 3, 20, 10), (6, 1, 64, 128), (2, 1, 72, 136), (4, 1, 128, 40), (8, 2, 32, 256)])
def test_differential_maps_and_their_join(dt, H, G, d, dv):
    """Both maps over a cache laid out head by head as [map 1, map 2], and their join, against one softmax per map; a key far away dominant in ONE of the two
    maps only (a swapped map, or one map's key read for the other, shows)."""
    from llm_quest_amd.common.mixers import differential_attention

    tol = 2e-5 if dt == "float32" else 3e-2
    scale, lam, eps, c = 0.25, 0.6, 1e-5, 0.5
    boosts = [(70, 0, (69, 0, 0)), (70, 0, (69, 0, 1)), (701, 700, (700, 63, 0)), (701, 700, (700, 320, 1)), (132, 129, (131, 64, 1))]
    for n, past, boost in [(n, p, None) for n, p in CASES] + boosts:
        q, k, v, qd, cache, desc = _kv_case(n, past, H, G, d, dv, dt, n + past, boost, maps=2)
        gate = torch.randn(n - past, H * dv, generator=torch.Generator().manual_seed(1))
        got = differential_attention(qd, cache, H, G, d, dv, scale, lam, eps, c, gate.to(DEV), desc, n - past, n, cache.dtype).double().cpu()
        for h in range(H):
            a1, a2 = (O.softmax_map(q[:, h, m], k[:, h // (H // G), m], v[:, h // (H // G)], scale)[past:] for m in (0, 1))
            want = O.unit_rms(a1 - lam * a2, eps) * c * torch.sigmoid(gate[:, h * dv : (h + 1) * dv].double())
            err = (got[:, h * dv : (h + 1) * dv] - want).pow(2).mean(-1).sqrt() / c
            assert float(err.max()) < tol, (n, past, boost, h)


def test_query_key_value_rows_with_fewer_value_heads():
    """Keys of 2 G map heads beside G value heads: the columns behind the keys are values, whatever their width."""
    from llm_quest_amd import kernels_seq as S

    g = torch.Generator().manual_seed(5)
    T, H, G, GV, d, dv, dims = 6, 6, 4, 2, 10, 14, 8
    src = torch.randn(T, (H + G) * d + GV * dv, generator=g)
    pos, rows = [3, 4, 5, 0, 1, 900], [7, 8, 9, 0, 1, 12]
    cache = torch.full((14, G * d + GV * dv), 5.0, device=DEV)
    q = S.qkv_rows_append(src.to(DEV), H, G, d, dv, None, None, None, 1e-5, None, dims, 0, S.rope_frequencies(dims, 70.0, DEV), dev_i32(pos), dev_i32(rows), cache, v_heads=GV)
    long_ = torch.zeros(901, H + G, d, dtype=F64)
    long_[pos] = src[:, : (H + G) * d].double().reshape(T, H + G, d)
    want = O.rotate(long_, dims, 70.0, True)[pos]
    assert torch.allclose(q.cpu().double(), want[:, :H].reshape(T, -1), atol=1e-3) and row_err(q, want[:, :H].reshape(T, -1)) < 1e-4
    assert row_err(cache[rows, : G * d], want[:, H:].reshape(T, -1)) < 1e-4 and torch.equal(cache[rows, G * d :].cpu(), src[:, (H + G) * d :])
    assert float((cache[[2, 3, 4, 5, 6, 10, 11, 13]] - 5.0).abs().max()) == 0.0


@pytest.mark.parametrize("C", [1, 60, 64, 130])
def test_minimal_gated_recurrence_in_steps(C):
    """Gates from nearly closed to nearly open, candidates on both sides of zero and exactly zero; three sequences in scattered slots, their states carried over
    portions that end inside and at the edges of the scan's 8- and 64-token tiles, and over single tokens."""
    from llm_quest_amd import kernels_seq as S

    g = torch.Generator().manual_seed(C)
    lens = [150, 31, 66]
    data = []
    for n in lens:
        z, u, gt = 4.0 * torch.randn(n, C, generator=g), torch.randn(n, C, generator=g), torch.randn(n, C, generator=g)
        u[::5] = 0.0
        z[n // 2] = 30.0
        z[n // 3] = -30.0
        data.append((z, u, gt))
    want = [O.min_gru_states(z.double(), u.double()) * gt.double() * torch.sigmoid(gt.double()) for z, u, gt in data]
    state = torch.full((5, C), 9.0, device=DEV)
    slots = [3, 0, 4]
    state[slots] = 0.0
    done, got = [0, 0, 0], [[], [], []]
    for cuts in ([64, 8, 1], [1, 1, 63], [71, 20, 2], [14, 2, 0]):
        live = [i for i in range(3) if cuts[i]]
        rows = [torch.cat([data[i][j][done[i] : done[i] + cuts[i]] for i in live]).to(DEV) for j in range(3)]
        both = torch.cat([rows[0], rows[1], rows[2]], dim=1)  # as the mixer passes them: views of one product
        off = [0]
        for i in live:
            off.append(off[-1] + cuts[i])
        out = S.mingru(both[:, :C], both[:, C : 2 * C], both[:, 2 * C :], dev_i32(off), dev_i32([slots[i] for i in live]), state, F32).cpu()
        for a, i in enumerate(live):
            got[i].append(out[off[a] : off[a + 1]])
            done[i] += cuts[i]
    for i, n in enumerate(lens):
        assert done[i] == n
        assert torch.allclose(torch.cat(got[i]).double(), want[i], atol=2e-5), i
    assert float((state[[1, 2]] - 9.0).abs().max()) == 0.0


def test_router_keeps_the_groups_with_the_largest_members():
    from llm_quest_amd import kernels_seq as S

    g = torch.Generator().manual_seed(4)
    for E, n, keep, top in ((12, 4, 3, 4), (8, 1, 1, 2), (70, 7, 3, 6), (6, 6, 3, 3), (5, 1, 1, 5), (130, 10, 4, 5), (512, 64, 9, 70), (4, 2, 1, 2), (1, 1, 1, 1)):
        logits = torch.randn(33, E, generator=g) * 2
        ids, wts = S.moe_route(logits.to(DEV), None, top, n, keep, 1.0, softmax=True)
        want_ids, want_w, gap = O.route(logits.double(), {"experts": E, "top": top, "groups": {"count": n, "keep": keep}})
        clear = gap > 1e-5
        assert int(clear.sum()) > 20
        assert torch.equal(ids.cpu().long()[clear].sort(1).values, want_ids[clear].sort(1).values), (E, n, keep, top)
        assert torch.allclose(wts.cpu().double().sort(1).values[clear], want_w[clear].sort(1).values, atol=2e-6)
        assert torch.allclose(wts.cpu().double()[clear].sum(1), want_w[clear].sum(1), atol=1e-5)  # the winners' own scores, not renormalised
    # the largest single score decides, not the largest pair
    ids, _ = S.moe_route(torch.tensor([[2.0, 2.0, 2.5, -5.0]], device=DEV), None, 1, 2, 1, 1.0, softmax=True)
    assert ids.tolist() == [[2]]


def test_logit_cap_rows():
    from llm_quest_amd import kernels_seq as S

    g = torch.Generator().manual_seed(0)
    for n in (64, 77):
        x = torch.randn(5, n + 3, generator=g).to(DEV)[:, 3:] * 20
        assert row_err(S.unary_rows(x, S.UNARY_SOFTCAP, limit=7.0), 7.0 * torch.tanh(x.double() / 7.0)) < 2e-6


def test_head_gate_sink_and_missing_rotation_of_latent_attention_keep_the_other_designs():
    """The latent mixer with a rotated part and an element-wise gate (its other users) still follows its own branch: parameters of the gate differ in size."""
    from llm_quest_amd.common.mixers import LatentAttention

    a = LatentAttention(32, 2, 8, 4, 6, 16, 12, 0.3, 4, 100.0, 1e-5, 0, gate=True)
    b = LatentAttention(32, 2, 8, 0, 6, 16, 12, 0.3, 0, 100.0, 1e-5, 0, gate="head", sink=True)
    assert a.w_down.shape[0] == 16 + 16 + 12 and b.w_down.shape[0] == 16 + 12 + 2 and a.sink is None and b.sink.numel() == 2
