"""GPU tests of the Pavisun serving path against the plain oracle (oracle/pavisun.py): each mechanism's kernel alone, then the model through the registry,
the slot cache and the ragged-batch scheduler -- whole prompts, token-by-token decoding, portions, unequal batches, reused slots, window edges, far keys, long
decoding, odd sizes, greedy generation, the trace replay program.  fp32 mode is held to fp32 rounding; bf16 mode to a few bf16 roundings of the logits' scale."""

import json
import os
import subprocess
import sys

import pytest
import torch

from oracle import pavisun as O
from tests import pavisun_util as U

pytestmark = pytest.mark.gpu
DEV = "cuda"
F32, F64, BF16, I32 = torch.float32, torch.float64, torch.bfloat16, torch.int32
TOL = {"float32": 3e-5, "bfloat16": 6e-2}
DTYPES = ["float32", "bfloat16"]
_oracle_cache = {}


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


def load(folder, cfg, w, dt):
    from llm_quest_amd import registry

    return registry.load_model(U.save(str(folder), cfg, w), dt, DEV)


@pytest.fixture(scope="module")
def checkpoint(tmp_path_factory):
    cfg = U.make_config(U.default_layers(), loop=(1, 3, 2))
    w = U.make_weights(cfg, 11)
    return U.save(str(tmp_path_factory.mktemp("pavisun")), cfg, w), cfg, w


@pytest.fixture(scope="module")
def models(checkpoint):
    from llm_quest_amd import registry

    folder, cfg, w = checkpoint
    return {dt: (registry.load_model(folder, dt, DEV), cfg, w) for dt in DTYPES}


def oracle(cfg, w, toks, layers=False):
    key = (id(w), str(cfg), tuple(toks), layers)
    if key not in _oracle_cache:
        _oracle_cache[key] = O.forward(cfg, w, toks, F64, return_layers=layers)
    return _oracle_cache[key]


def batch_of(model, **kw):
    from llm_quest_amd.generate import RaggedBatch

    return RaggedBatch(model, **kw)


# ------------------------------------------------------------------------------------------------------------------- the model through the scheduler
@pytest.mark.parametrize("dt", DTYPES)
def test_whole_prompt_every_layer_run(models, dt):
    model, cfg, w = models[dt]
    toks = tokens(70, cfg["vocab"], 1)
    want, layers = oracle(cfg, w, toks, layers=True)
    got, got_layers = batch_of(model).step([("a", toks)], [list(range(len(toks)))], return_layers=True)
    assert len(got_layers) == len(layers) == 7
    for i, l in enumerate(got_layers):
        assert row_err(l, layers[i]) < TOL[dt], f"streams after layer run {i}"
    assert row_err(got, want) < TOL[dt]


@pytest.mark.parametrize("dt", DTYPES)
def test_token_by_token_from_the_first_token(models, dt):
    model, cfg, w = models[dt]
    toks = tokens(60, cfg["vocab"], 2)
    b = batch_of(model)
    got = torch.cat([b.step([("a", [t])]) for t in toks])
    assert row_err(got, oracle(cfg, w, toks)) < TOL[dt]


@pytest.mark.parametrize("dt", DTYPES)
def test_portions_of_several_sizes(models, dt):
    """Portions down to one and two tokens: the first is a prompt, the others go on against the cache."""
    model, cfg, w = models[dt]
    toks = tokens(95, cfg["vocab"], 3)
    b = batch_of(model)
    got, at = [], 0
    for n in [7, 2, 2, 1, 1, 33, 1, 9, 2, 32, 5]:
        got.append(b.step([("a", toks[at : at + n])], [list(range(n))]))
        at += n
    assert at == len(toks)
    assert row_err(torch.cat(got), oracle(cfg, w, toks)) < TOL[dt]


@pytest.mark.parametrize("dt", DTYPES)
def test_unequal_batch_equals_each_request_alone(models, dt):
    model, cfg, w = models[dt]
    lens, tail = [1, 41, 17, 66], 9
    seqs = [tokens(n + tail, cfg["vocab"], 10 + i) for i, n in enumerate(lens)]
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
        assert row_err(g, alone[i][: g.shape[0]]) < (1e-5 if dt == "float32" else 5e-2), f"request {i} in the batch differs from the request alone"
        assert row_err(g, oracle(cfg, w, s)[: g.shape[0]]) < TOL[dt]


def test_mixed_batch_of_prompts_portions_and_single_tokens(models):
    """One step holds a new prompt, a portion of an older one and a single token of a third; each equals the request alone."""
    model, cfg, w = models["float32"]
    seqs = [tokens(n, cfg["vocab"], 60 + n) for n in (40, 35, 30)]
    b = batch_of(model)
    got = {0: [b.step([(0, seqs[0][:25])], [list(range(25))])], 1: [], 2: []}
    for step in [[(0, 25, 26), (1, 0, 20)], [(0, 26, 39), (1, 20, 21), (2, 0, 28)], [(1, 21, 35), (0, 39, 40), (2, 28, 30)]]:
        out = b.step([(i, seqs[i][a:e]) for i, a, e in step], [list(range(e - a)) for _, a, e in step])
        at = 0
        for i, a, e in step:
            got[i].append(out[at : at + e - a])
            at += e - a
    for i, s in enumerate(seqs):
        assert row_err(torch.cat(got[i]), oracle(cfg, w, s)) < TOL["float32"], i


@pytest.mark.parametrize("dt", DTYPES)
def test_freed_slots_are_reused_without_leftovers(models, dt):
    """A long sequence leaves key / value rows behind in every pass's cache; the next, shorter one takes its slot and must see none of them.  The cache starts small, so
    rows also grow while a sequence is alive."""
    model, cfg, w = models[dt]
    b = batch_of(model, slots=1)
    b.cache.initial_chunk_size, b.cache.chunk_size = 4, 8
    long_, short = tokens(60, cfg["vocab"], 20), tokens(33, cfg["vocab"], 21)
    b.step([("long", long_[:50])])
    for t in long_[50:]:
        b.step([("long", [t])])
    b.finish("long")
    got = [b.step([("short", short[:12])], [list(range(12))])] + [b.step([("short", [t])]) for t in short[12:]]
    assert b.cache.reuses >= 1 and b.cache.slots == 1
    assert row_err(torch.cat(got), oracle(cfg, w, short)) < TOL[dt]


def test_long_decoding(models):
    """220 decoded tokens: every window slides far past what was prefilled, the kept first tokens stay."""
    model, cfg, w = models["float32"]
    toks = tokens(225, cfg["vocab"], 30)
    b = batch_of(model)
    b.step([("a", toks[:5])])
    got = torch.cat([b.step([("a", [t])]) for t in toks[5:]])
    assert row_err(got, oracle(cfg, w, toks)[5:]) < TOL["float32"]


@pytest.mark.parametrize("dt", DTYPES)
def test_long_prompt_then_decoding_with_dealt_out_keys(tmp_path, dt):
    """Windows of hundreds of keys: one-token steps deal a tile's keys (kept ones too) to several workgroups whose partial results meet.  A shorter request beside the long
    one leaves most shares of the deal empty."""
    cfg = U.make_config([(U.attention(size=600), None), (U.attention_2(heads=4, size=530, keep_first=70, scale=0.5), None), (U.attention(size=2000, scaling=None, softcap=0.0), None)])
    w = U.make_weights(cfg, 3)
    model = load(tmp_path, cfg, w, dt)
    toks, other = tokens(904, cfg["vocab"], 4), tokens(97, cfg["vocab"], 5)
    want, want2 = oracle(cfg, w, toks), oracle(cfg, w, other)
    b = batch_of(model)
    got = b.step([("a", toks[:897]), ("b", other[:90])], [[0, 1, 600, 601, 896], [89]])
    assert row_err(got[:5], want[[0, 1, 600, 601, 896]]) < TOL[dt] and row_err(got[5:], want2[89:90]) < TOL[dt]
    got = torch.stack([b.step([("a", [t]), ("b", [u])]) for t, u in zip(toks[897:], other[90:])])
    assert row_err(got[:, 0], want[897:]) < TOL[dt] and row_err(got[:, 1], want2[90:]) < TOL[dt]


@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("kind,size,keep", [("attention", 1, 0), ("attention", 13, 0), ("attention", 64, 0), ("attention_2", 11, 5), ("attention_2", 64, 1), ("attention_2", 3, 64), ("attention_2", 20, 66),
                                            ("attention_2", 9, 0)])
@pytest.mark.parametrize("dt", DTYPES)
def test_a_token_counts_exactly_where_it_is_seen(tmp_path, dt, kind, size, keep, decoded):
    """One layer: changing ONE token of the sequence changes the logits of exactly those later positions whose window (or kept first tokens) holds it, in prompts and
    in decoding; everywhere else they are the same bit for bit."""
    mixer = U.attention(size=size, softcap=30.0) if kind == "attention" else U.attention_2(size=size, keep_first=keep, scale=0.5)
    cfg = U.make_config([(mixer, None)], vocab=50)
    w = U.make_weights(cfg, 8)
    model = load(tmp_path, cfg, w, dt)
    n = 140
    base = tokens(n, 50, 9)
    m = 70 if decoded else n

    def run(toks):
        b = batch_of(model)
        out = [b.step([("a", toks[:m])], [list(range(m))])]
        return torch.cat(out + [b.step([("a", [t])]) for t in toks[m:]])

    ref = run(base)
    for j in (0, 1, keep - 1, keep, 60, 63, 64):
        if not 0 <= j < n:
            continue
        other = list(base)
        other[j] = (base[j] + 7) % 50
        same = (run(other) == ref).all(dim=1).cpu()
        i = torch.arange(n)
        seen = (i >= j) & ((i - j < size) | torch.tensor(j < keep))
        if kind == "attention_2":  # the distance bias makes far kept tokens vanish in rounding: near ones must show
            assert bool(same[~seen].all()), (j, "a hidden token counts")
            near = seen & (i - j < 12)
            assert not bool(same[near].any()), (j, "a visible token does not count")
        else:
            assert torch.equal(~same, seen), j


def test_passes_of_a_loop_keep_their_own_keys(tmp_path):
    """Loops of one, two and three passes, over the first, the middle, the last and all layers: prompt, then decoding through the caches of every pass."""
    layers = [(U.attention(), U.moe()), (U.attention_2(), None), (U.attention(heads=2, kv_heads=1), U.moe(top=1))]
    for k, loop in enumerate([(0, 1, 2), (1, 2, 3), (2, 3, 2), (0, 3, 2), (1, 3, 1), (1, 1, 4)]):
        cfg = U.make_config(layers, loop=loop)
        w = U.make_weights(cfg, 40 + k)
        model = load(tmp_path / str(k), cfg, w, "float32")
        assert len(model.cfg.runs) == 3 + (loop[1] - loop[0]) * (loop[2] - 1)
        toks = tokens(40, cfg["vocab"], 41 + k)
        b = batch_of(model)
        got = [b.step([("a", toks[:20])], [list(range(20))])] + [b.step([("a", [t])]) for t in toks[20:]]
        assert row_err(torch.cat(got), oracle(cfg, w, toks)) < TOL["float32"], loop


@pytest.mark.parametrize("dt", DTYPES)
def test_other_sizes_odd_and_one(tmp_path, dt):
    """Sizes that are no multiples of 8 or of each other's: one stream and nine, one head, one key head per query head, a rotation of two entries and of none, heads of odd
    width, windows of one key and wider than the sequence, nothing kept and more kept than there is, one expert, every expert, no caps, no feed-forward anywhere."""
    stacks = [(dict(width=100, vocab=77, eps=1e-6, streams=1, softcap=0.0, loop=(0, 2, 2)),
               [(U.attention(heads=1, kv_heads=1, dim=7, size=1, rot_dims=2, base=3.0, scaling=(2.0, 30, 3.0, 0.2)), U.moe(experts=1, top=1, ff=20)),
                (U.attention_2(heads=5, kv_heads=1, dim=3, vdim=41, size=6, keep_first=0, scale=0.7), U.moe(experts=4, top=4, ff=33)),
                (U.attention(heads=3, kv_heads=1, dim=14, size=500, rot_dims=0, softcap=0.0), U.moe(experts=9, top=3, ff=7))]),
              (dict(width=33, vocab=40, streams=9, softcap=3.0),
               [(U.attention_2(heads=7, kv_heads=7, dim=9, vdim=1, size=2, keep_first=100, scale=0.8), None),
                (U.attention(heads=2, kv_heads=2, dim=6, size=3, rot_dims=6, base=3.0, scaling=(1.0, 12, 9.0, 0.1)), U.moe(experts=70, top=5, ff=12))]),
              (dict(width=64, vocab=64, streams=2), [(U.attention_2(heads=1, kv_heads=1, dim=1, vdim=5, size=1, keep_first=1), None), (U.attention(heads=4, kv_heads=1, size=48), None)])]
    for k, (kw, layers) in enumerate(stacks):
        cfg = U.make_config(layers, **kw)
        w = U.make_weights(cfg, 5 + k)
        model = load(tmp_path / str(k), cfg, w, dt)
        toks = tokens(48, cfg["vocab"], 6)
        b = batch_of(model)
        got = [b.step([("a", toks[:29])], [list(range(29))]), b.step([("a", toks[29:31])], [[0, 1]])] + [b.step([("a", [t])]) for t in toks[31:]]
        assert row_err(torch.cat(got), oracle(cfg, w, toks)) < TOL[dt], k


@pytest.mark.parametrize("dt", DTYPES)
def test_wide_rows_and_wide_heads(tmp_path, dt):
    """Rows wider than 512 on five streams, heads of 136, 200 and 264 (beyond what the MFMA kernel keeps in registers), values of 72 and 264."""
    layers = [(U.attention(heads=2, kv_heads=1, dim=136, rot_dims=64, size=20), U.moe(ff=64)), (U.attention_2(heads=2, kv_heads=2, dim=200, vdim=72, size=17, scale=0.12), None),
              (U.attention(heads=2, kv_heads=1, dim=264, rot_dims=264, size=9), None), (U.attention_2(heads=4, kv_heads=2, dim=24, vdim=264, size=12, keep_first=3, scale=0.4), U.moe(experts=3, top=1, ff=520))]
    cfg = U.make_config(layers, width=520, vocab=50, streams=5)
    w = U.make_weights(cfg, 9)
    model = load(tmp_path, cfg, w, dt)
    toks = tokens(40, cfg["vocab"], 8)
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


@pytest.mark.parametrize("dt", DTYPES)
def test_trace_replay_program_end_to_end(checkpoint, tmp_path, dt):
    """bin/trace_run as a user runs it: a folder, steps on standard input (two prompts in one batch, then one token each, one request ending early and
    its slot taken by a third), logits files out -- against the oracle."""
    import numpy as np

    folder, cfg, w = checkpoint
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    a, b, c = tokens(31, cfg["vocab"], 50), tokens(9, cfg["vocab"], 51), tokens(12, cfg["vocab"], 52)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:28], "want": [0, 13, 27]}, {"id": "b", "tokens": b[:8], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[28:29], "want": [0]}, {"id": "b", "tokens": b[8:9], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[29:30], "want": []}], "end": []},
             {"step": 3, "entries": [{"id": "c", "tokens": c, "want": [11]}], "end": ["c"]},
             {"step": 4, "entries": [{"id": "a", "tokens": a[30:31], "want": [0]}], "end": ["a"]}]
    wa, wb, wc = oracle(cfg, w, a), oracle(cfg, w, b), oracle(cfg, w, c)
    want = {0: torch.stack([wa[0], wa[13], wa[27]]), 1: torch.stack([wa[28], wb[8]]), 3: wc[11:12], 4: wa[30:31]}
    out = tmp_path / "out"
    res = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", dt, "--out", str(out), "--max-tokens", "64"],
                         input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=100)
    assert res.returncode == 0, res.stderr[-2000:]
    assert [l for l in res.stdout.split("\n") if l.startswith("done")] == [f"done {i}" for i in range(5)]
    assert not (out / "2.f32").exists()
    for i, ref in want.items():
        got = torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, cfg["vocab"]))
        assert got.shape == ref.shape and row_err(got, ref) < TOL[dt], (dt, i)


# ------------------------------------------------------------------------------------------------------------------- mechanisms alone
@pytest.mark.parametrize("S", [1, 2, 3, 4, 5, 8, 11])
@pytest.mark.parametrize("width", [72, 33, 256, 500, 1000, 2048, 4100])
def test_streams_join_mix_and_read(S, width):
    from llm_quest_amd import kernels_seq as K

    g = torch.Generator().manual_seed(width + S)
    T, parts, eps = 9, 3, 1e-4
    r = lambda *s: torch.randn(*s, generator=g)
    d = lambda t: t.to(DEV)
    xs, y1, y3, mix, put, read, nw = r(T, S, width), r(T, width), r(T * parts, width + 4), r(S, S), r(S), r(S), 1.0 + 0.3 * r(width)
    read = read * torch.where(torch.arange(S) == 0, 0.05, 1.0) * 0.05  # eps counts in the norm
    norm = lambda u: u / torch.sqrt((u * u).mean(-1, keepdim=True) + eps) * nw.double()
    for ydt in (F32, BF16):
        a = y3.to(ydt)
        yv = a[:, :width].double().reshape(T, parts, width).sum(1) / parts
        new = torch.stack([sum(mix[s, t].double() * xs[:, s].double() for s in range(S)) + put[t].double() * yv for t in range(S)], dim=1)
        u = sum(read[s].double() * new[:, s] for s in range(S))
        old = d(xs)
        x_out, h, uu = K.hyper_mix(old, S, y=d(a)[:, :width], parts=parts, y_scale=1.0 / parts, mix=d(mix), put=d(put), read=d(read), x_out=True, want_u=True, norm=d(nw), eps=eps, out_dtype=F32)
        assert torch.allclose(x_out.cpu().double(), new, atol=3e-5) and torch.allclose(uu.cpu().double(), u, atol=1e-5) and row_err(h, norm(u)) < 1e-5
        assert torch.equal(old.cpu(), xs)
        _, hb, _ = K.hyper_mix(old, S, y=d(a)[:, :width], parts=parts, y_scale=1.0 / parts, mix=d(mix), put=d(put), read=d(read), norm=d(nw), eps=eps, out_dtype=BF16)
        assert torch.equal(hb.cpu(), h.cpu().to(BF16))
        # some tokens only, in an order of their own
        rows = torch.tensor([7, 0, 8, 8, 3])
        xr, hr, _ = K.hyper_mix(old, S, y=d(a)[:, :width], parts=parts, y_scale=1.0 / parts, mix=d(mix), put=d(put), read=d(read), rows=d(rows), x_out=True, norm=d(nw), eps=eps, out_dtype=F32)
        assert torch.equal(xr, x_out[d(rows)]) and torch.equal(hr, h[d(rows)])
    # all streams alike: read off one row; nothing pending; and a first join onto them
    none, h, uu = K.hyper_mix(d(y1), S, read=d(read), want_u=True, norm=d(nw), eps=eps, out_dtype=F32)
    assert none is None and row_err(uu, y1.double() * read.double().sum()) < 1e-5 + 1e-6 / abs(float(read.sum())) and row_err(h, norm(y1.double() * float(read.double().sum()))) < 1e-4
    x_out, _, _ = K.hyper_mix(d(y1), S, y=d(y3[:T, :width].contiguous()), mix=d(mix), put=d(put), x_out=True)
    want = mix.double().sum(0)[None, :, None] * y1.double()[:, None] + put.double()[None, :, None] * y3[:T, :width].double()[:, None]
    assert torch.allclose(x_out.cpu().double(), want, atol=3e-5)


@pytest.mark.parametrize("T", [1, 7, 64, 1000, 9001])
def test_dispatch_lists_from_tables_and_from_ids(T):
    """Entries sorted by expert, in token order inside one; every layer of a step in one launch, layers of different expert counts and choices side by side."""
    from llm_quest_amd import kernels_seq as K

    g = torch.Generator().manual_seed(T)
    vocab, specs = 300, [(2, 5), (1, 1), (6, 130), (3, 3), (4, 2100)]
    tok = torch.randint(0, vocab, (T,), generator=g)
    tables = [torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(vocab)]) for top, E in specs]
    meta, at = [], 0
    for (top, E), t in zip(specs, tables):
        meta += [at, top, E, 0]
        at += t.numel()
    lists = K.moe_table_dispatch(tok.to(I32).to(DEV), vocab, torch.cat([t.reshape(-1) for t in tables]).to(I32).to(DEV), dev_i32(meta), specs)
    for (top, E), t, (offs, perm) in zip(specs, tables, lists):
        ids = t[tok].reshape(-1)
        want = torch.argsort(ids, stable=True)
        counts = torch.bincount(ids, minlength=E)
        for o, p in ((offs, perm), K.moe_dispatch(ids.to(I32).to(DEV), E)):
            assert torch.equal(o.cpu().long(), torch.cat([torch.zeros(1, dtype=torch.long), counts.cumsum(0)])), (top, E)
            assert torch.equal(p.cpu().long(), want), (top, E)


def test_dispatch_of_many_entries_over_many_rounds():
    """More entries than the sort keeps in registers between its passes, most of them of one expert."""
    from llm_quest_amd import kernels_seq as K

    g = torch.Generator().manual_seed(1)
    for n, E in ((70001, 16), (40000, 3000), (20000, 1)):
        ids = torch.where(torch.rand(n, generator=g) < 0.7, torch.tensor(E // 2), torch.randint(0, E, (n,), generator=g))
        offs, perm = K.moe_dispatch(ids.to(I32).to(DEV), E)
        assert torch.equal(perm.cpu().long(), torch.argsort(ids, stable=True)) and int(offs[-1]) == n
        assert torch.equal(offs.cpu().long()[1:], torch.bincount(ids, minlength=E).cumsum(0))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("experts,top,ff", [(6, 2, 40), (1, 1, 24), (5, 5, 33), (40, 3, 64)])
def test_table_experts_alone(dt, experts, top, ff):
    """Every token id's own experts, equal weights; the sum over a token's rows times 1 / top is what the oracle adds."""
    from llm_quest_amd.common.mixers import SeqStep, TableMoE
    from llm_quest_amd.utils import SlotStateCache

    cfg = U.make_config([(U.attention(), U.moe(experts, top, ff))], vocab=30)
    w = U.make_weights(cfg, experts)
    ff_ = TableMoE(cfg["width"], ff, experts, top, 30)
    ff_.load_table(w["l0.mlp.table"])
    ff_.load_experts(*[[w[f"l0.mlp.e{j}.{s}"] for j in range(experts)] for s in ("gate", "up", "down")])
    ff_ = ff_.to(DEV)
    act = torch.float32 if dt == "float32" else BF16
    toks = tokens(50, 30, 3)
    st = SeqStep(_cache_with_slot(SlotStateCache([None], 4096, DEV, act)), [(0, toks)], DEV, act)
    h = torch.randn(50, cfg["width"], generator=torch.Generator().manual_seed(4)).to(act)
    out = ff_.step(h.to(DEV), TableMoE.dispatch(TableMoE.gather_tables([ff_]), st)[0])
    d = {k: v.double() if v.is_floating_point() else v for k, v in w.items()}
    want = O.table_experts(h.double(), toks, d, "l0.mlp.", cfg["layers"][0]["mlp"])
    assert row_err(out.reshape(50, top, -1).sum(1) / top, want) < (3e-6 if dt == "float32" else 2e-2)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("width,ff,experts,top", [(264, 520, 5, 2), (512, 300, 3, 1), (260, 256, 4, 3), (1024, 64, 9, 2)])
def test_experts_of_every_number_of_rows(dt, width, ff, experts, top):
    """From one token (the weights are streamed) to hundreds (tiles): one expert taking nearly every row, one taking none, widths that are multiples of 8 and not; a
    token's rows do not depend on how many others there are, beyond rounding."""
    from llm_quest_amd import kernels_seq as K
    from llm_quest_amd.common.mixers import TableMoE

    g = torch.Generator().manual_seed(width + ff)
    r = lambda *s: (torch.randn(*s, generator=g) / s[-1] ** 0.5).to(BF16)
    gates, ups, downs = [r(ff, width) for _ in range(experts)], [r(ff, width) for _ in range(experts)], [r(width, ff) for _ in range(experts)]
    m = TableMoE(width, ff, experts, top, 1)
    m.load_experts(gates, ups, downs)
    m = m.to(DEV)
    act = F32 if dt == "float32" else BF16
    h = torch.randn(400, width, generator=g).to(act)
    score = torch.rand(400, experts, generator=g) + torch.tensor([2.0 * (e == 1) - 5.0 * (e == 0 and top < experts) for e in range(experts)])
    ids = score.argsort(dim=1, descending=True)[:, :top]
    want = torch.empty(400, top, width, dtype=F64)
    for e in range(experts):
        z = h.double() @ gates[e].double().T
        y = (z * torch.sigmoid(z) * (h.double() @ ups[e].double().T)) @ downs[e].double().T
        want[ids == e] = y[(ids == e).any(1)]
    for T in (1, 2, 33, 85, 130, 400):
        offs, perm = K.moe_dispatch(ids[:T].reshape(-1).to(I32).to(DEV), experts)
        wts = None if T % 2 else torch.rand(T, top, generator=g)
        out = m.run_experts(h[:T].to(DEV), offs, perm, None if wts is None else wts.to(DEV)).reshape(T, top, width)
        ref = want[:T] if wts is None else want[:T] * wts.double()[..., None]
        assert float((out.cpu().double() - ref).abs().max()) < (2e-5 if dt == "float32" else 2e-2) * float(want.abs().max()), T


def _cache_with_slot(cache):
    cache.open("s")
    return cache


@pytest.mark.parametrize("T", [5, 400])
@pytest.mark.parametrize("H,G,d,dims", [(4, 2, 24, 16), (3, 3, 10, 10), (6, 1, 128, 64), (2, 1, 7, 2), (4, 2, 64, 0), (16, 2, 128, 128), (2, 2, 264, 200), (5, 5, 20, 12)])
def test_query_key_rows_with_tied_values_unit_norms_and_an_amplitude(H, G, d, dims, T):
    """Values that are the keys before rotation (and before a norm); unit-RMS heads where eps counts; cosine and sine times an amplitude; the same with own values."""
    from llm_quest_amd import kernels_seq as K

    g = torch.Generator().manual_seed(d + T)
    eps, amp = 1e-3, 1.3
    pos = torch.randperm(T + 300, generator=g)[:T]
    rows = torch.randperm(T + 40, generator=g)[:T]
    freqs = [float(300.0 ** (-2.0 * i / max(dims, 1))) for i in range(dims // 2)]
    freq = torch.tensor(freqs, dtype=F32).to(DEV) if dims else None
    qs = 0.5 + torch.rand(H, generator=g)

    def rot(x):  # [T, heads, d] at their positions
        if not dims:
            return x
        ang = pos.double()[:, None] * torch.tensor(freqs, dtype=F32).double()[None]
        c, s = torch.cos(ang)[:, None] * amp, torch.sin(ang)[:, None] * amp
        u, v = x[..., : dims // 2], x[..., dims // 2 : dims]
        return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], dim=-1)

    for tied in (True, False):
        dv = d if tied else d + 4
        src = torch.randn(T, (H + G) * d + (0 if tied else G * dv) + 3, generator=g)
        src[:, :d] *= 0.02
        n = src.shape[1] - 3
        q0, k0 = src[:, : H * d].double().reshape(T, H, d), src[:, H * d : (H + G) * d].double().reshape(T, G, d)
        v0 = k0.reshape(T, -1) if tied else src[:, (H + G) * d : n].double()
        for unit in (False, True):
            norm = (lambda x: O.unit_rms(x, eps)) if unit else (lambda x: x)
            for layout in (1,) if dims else (0, 1):
                cache = torch.full((T + 40, G * (d + dv)), 5.0, device=DEV)
                q = K.qkv_rows_append(src.to(DEV)[:, :n], H, G, d, dv, None, None, None, eps, qs.to(DEV), dims, layout, freq, pos.to(I32).to(DEV), rows.to(I32).to(DEV), cache,
                                      unit_norm=unit, rot_amp=amp, tie_v=tied)
                assert row_err(q, (rot(norm(q0)) * qs.double()[None, :, None]).reshape(T, -1)) < 2e-5
                got = cache.cpu()[rows]
                assert row_err(got[:, : G * d], rot(norm(k0)).reshape(T, -1)) < 2e-5 and torch.equal(got[:, G * d :].double(), v0)
                left = torch.ones(T + 40, dtype=torch.bool)
                left[rows] = False
                assert float((cache.cpu()[left] - 5.0).abs().max()) == 0.0


def _kv_case(n, past, H, G, d, dv, dt, seed, boost=None):
    """fp32 queries [n_new, H * d] and a cache [G x d | G x dv] of n rows behind five foreign rows.  ``boost`` = (query position, key position): that query and key are made
    parallel and long, so that the key dominates the row."""
    g = torch.Generator().manual_seed(seed)
    q, k, v = torch.randn(n, H, d, generator=g), torch.randn(n, G, d, generator=g), torch.randn(n, G, dv, generator=g)
    if boost:
        qi, kj = boost
        q[qi] = 4.0 * k[kj].repeat_interleave(H // G, dim=0)
        k[kj] = 3.0 * k[kj]
        v[kj] = 30.0 * v[kj]
    kv_dt = BF16 if dt == "bfloat16" else F32
    k, v = k.to(kv_dt), v.to(kv_dt)
    cache = torch.full((5 + n + 3, G * (d + dv)), 7.0, dtype=kv_dt, device=DEV)
    cache[5 : 5 + n] = torch.cat([k.reshape(n, -1), v.reshape(n, -1)], dim=1).to(DEV)
    desc = (dev_i32([0]), dev_i32([n - past]), dev_i32([past]), dev_i32([5]), dev_i32([5]), dev_i32([5]))
    return q.double(), k.double(), v.double(), q[past:].reshape(n - past, -1).contiguous().to(DEV), cache, desc


def _attn_check(case, H, G, d, dv, scale, size, keep, cap, slopes, gate, tol, where):
    from llm_quest_amd import kernels_seq as K
    from llm_quest_amd.common.mixers import _largest_pow2_divisor

    q, k, v, qd, cache, desc = case
    n, past = q.shape[0], q.shape[0] - qd.shape[0]
    out = torch.empty(n - past, H * dv, dtype=cache.dtype, device=DEV)
    sl = None if slopes is None else torch.tensor(slopes, dtype=F32).to(DEV)
    gt = None if gate is None else gate[past:n].to(DEV)
    K.latent_attn(qd, cache, None, cache[:, G * d :], out, H, _largest_pow2_divisor(H // G), d, 0, dv, d, d, dv, dv, desc, n - past, scale, max_keys=n, kv_rep=H // G, window=size,
                  keep_first=keep, softcap=cap, slope=sl, gate=gt)
    ok = O.visible(n, size, keep)
    for h in range(H):
        want = O.softmax_head(q[:, h], k[:, h // (H // G)], v[:, h // (H // G)], scale, ok, cap, 0.0 if slopes is None else slopes[h])[past:]
        if gate is not None:
            want = want * torch.sigmoid(gate[past:n, h * dv : (h + 1) * dv].double())
        got = out[:, h * dv : (h + 1) * dv].double().cpu()
        assert float((got - want).abs().max()) < tol * max(float(want.abs().max()), 1.0), (where, h)


# (keys, of which cached, window, kept, boosted (query, key)): prompts, portions, one-token steps; keys just inside and just outside the window and the kept tokens,
# around the kernels' 64-key steps
WINDOW_CASES = [(70, 0, 13, 0, None), (200, 0, 64, 5, None), (127, 37, 50, 3, None), (701, 700, 300, 20, None), (1500, 1499, 700, 130, None), (132, 129, 40, 64, None), (15, 10, 4, 2, None),
                (64, 0, 1, 0, None), (65, 64, 64, 0, None), (1, 0, 5, 3, None), (300, 0, 100, 300, None), (900, 880, 128, 1, None), (260, 0, 0, 0, None), (513, 512, 0, 0, None),
                (70, 0, 13, 0, (69, 57)), (70, 0, 13, 0, (69, 56)), (70, 0, 13, 5, (69, 4)), (70, 0, 13, 5, (69, 5)), (200, 0, 64, 0, (191, 128)), (200, 0, 64, 0, (191, 127)),
                (701, 700, 300, 20, (700, 401)), (701, 700, 300, 20, (700, 400)), (701, 700, 300, 20, (700, 19)), (701, 700, 300, 20, (700, 20)), (701, 700, 300, 64, (700, 63)),
                (701, 700, 300, 64, (700, 64)), (132, 129, 40, 65, (131, 64)), (132, 129, 40, 65, (131, 65)), (132, 129, 40, 65, (131, 92)), (132, 129, 40, 65, (131, 91)), (1500, 1499, 0, 0, (1499, 3))]


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,d,dv", [(4, 2, 24, 40), (6, 2, 16, 16), (3, 1, 20, 12)])
def test_windows_with_kept_tokens_caps_biases_and_gates(dt, H, G, d, dv):
    """(4, 2) and (6, 2): aligned rows, the lean MFMA kernel in bf16; (3, 1) with widths of 20 and 12: the general one."""
    tol = 2e-5 if dt == "float32" else 4e-2
    slopes = [2.0 ** (-8.0 * (h + 1) / H) for h in range(H)]
    gate = torch.randn(1500, H * dv, generator=torch.Generator().manual_seed(2)) * 2
    for n, past, size, keep, boost in WINDOW_CASES:
        case = _kv_case(n, past, H, G, d, dv, dt, n + past, boost)
        for cap, sl, gt in ((0.0, None, None), (2.0, None, None), (0.0, [s * 0.1 for s in slopes], gate), (1.5, [s * 0.02 for s in slopes], gate), (0.0, None, gate)):
            _attn_check(case, H, G, d, dv, 0.3, size, keep, cap, sl, gt, tol, (n, past, size, keep, boost, cap, sl is not None))


def test_a_real_distance_bias_far_away():
    """Slopes as the design has them: kept first tokens hundreds of positions away still show for the heads with small slopes, and differences of the bias between
    neighbouring keys stay exact at large distances."""
    H, G, d, dv = 8, 2, 32, 32
    slopes = [2.0 ** (-8.0 * (h + 1) / H) for h in range(H)]
    for dt in DTYPES:
        for n, past, size, keep, boost in ((3001, 3000, 50, 8, (3000, 7)), (3001, 3000, 50, 8, (3000, 2951)), (3001, 2990, 2000, 8, None), (400, 0, 50, 8, (399, 2))):
            case = _kv_case(n, past, H, G, d, dv, dt, n + size, boost)
            _attn_check(case, H, G, d, dv, 0.3, size, keep, 0.0, slopes, None, 3e-5 if dt == "float32" else 2e-2, (dt, n, past, size, boost))


@pytest.mark.parametrize("D,DV", [(64, 32), (72, 72), (128, 128), (128, 200), (192, 128), (200, 96), (256, 128), (256, 256), (264, 64), (96, 264)])
def test_windows_at_every_width(D, DV):
    """Every width class of the kernels, three sequences of unequal lengths in one launch (prompt, portions, one-token steps), window and kept tokens, with and without cap
    and bias."""
    from llm_quest_amd import kernels_seq as K

    g = torch.Generator().manual_seed(D + DV)
    H, scale, size, keep = 2, D ** -0.5, 70, 3
    slopes = [0.05, 0.004]
    gate_all = torch.randn(400, H * DV, generator=g)
    for new, past in (([70, 5, 129], [0, 0, 0]), ([1, 1, 1], [600, 3, 64]), ([2, 33, 1], [90, 31, 63])):
        q = torch.randn(sum(new), H * D, generator=g) * 2
        n = [a + b for a, b in zip(new, past)]
        cap_rows = max(n) + 4
        k, v = (torch.randn(3 * cap_rows, H * w_, generator=g).to(BF16) for w_ in (D, DV))
        q_row0, row0 = [0, new[0], new[0] + new[1]], [cap_rows * i for i in range(3)]
        desc = tuple(dev_i32(t) for t in (q_row0, new, past, row0, row0, row0))
        for softcap, sl in ((0.0, None), (3.0, slopes)):
            for o_dt in (F32, BF16):
                out = torch.zeros(sum(new), H * DV, dtype=o_dt, device=DEV)
                K.latent_attn(q.to(DEV), k.to(DEV), None, v.to(DEV), out, H, 1, D, 0, DV, D, D, DV, DV, desc, max(new), scale, max_keys=max(n), window=size, keep_first=keep, softcap=softcap,
                              slope=None if sl is None else torch.tensor(sl).to(DEV), gate=gate_all[: sum(new)].to(DEV))
                for s in range(3):
                    rows = slice(row0[s], row0[s] + n[s])
                    for h in range(H):
                        qq = torch.zeros(n[s], D, dtype=F64)
                        qq[past[s] :] = q[q_row0[s] : q_row0[s] + new[s], h * D : (h + 1) * D].double()
                        want = O.softmax_head(qq, k[rows, h * D : (h + 1) * D].double(), v[rows, h * DV : (h + 1) * DV].double(), scale, O.visible(n[s], size, keep), softcap, sl[h] if sl else 0.0)[past[s] :]
                        want = want * torch.sigmoid(gate_all[q_row0[s] : q_row0[s] + new[s], h * DV : (h + 1) * DV].double())
                        got = out[q_row0[s] : q_row0[s] + new[s], h * DV : (h + 1) * DV].double().cpu()
                        assert float((got - want).abs().max()) < 3e-2 * float(want.abs().max()), (new, past, s, h, o_dt, softcap)
