"""CPU checks around the Pavisun serving path: the oracle's mechanisms against independent restatements, the configuration parser, the checkpoint loader's
fused parameters and the cache layout.  Nothing here needs a GPU."""

import math

import pytest
import torch

from oracle import pavisun as O
from tests import pavisun_util as U

F64 = torch.float64


def test_oracle_prefix_property():
    """Logits at a position depend on the tokens up to it only: a prefix gives the same rows."""
    cfg = U.make_config(U.default_layers(), loop=(1, 3, 2))
    w = U.make_weights(cfg, 1)
    g = torch.Generator().manual_seed(0)
    toks = torch.randint(0, cfg["vocab"], (30,), generator=g).tolist()
    full = O.forward(cfg, w, toks, F64)
    part = O.forward(cfg, w, toks[:17], F64)
    assert torch.allclose(full[:17], part, atol=1e-10)
    assert float(full.abs().max()) <= cfg["logit_softcap"]


def test_oracle_attention_closed_forms():
    g = torch.Generator().manual_seed(1)
    q, k, v = (torch.randn(15, n, generator=g, dtype=F64) for n in (6, 6, 4))
    for size, keep in ((5, 0), (1, 0), (4, 3), (3, 7), (40, 2), (0, 0)):
        for cap, slope in ((0.0, 0.0), (1.5, 0.0), (0.0, 0.3)):
            ok = O.visible(15, size, keep)
            got = O.softmax_head(q, k, v, 0.4, ok, cap, slope)
            for i in range(15):
                seen = [j for j in range(i + 1) if size == 0 or i - j < size or j < keep]
                s = [float(q[i] @ k[j]) * 0.4 for j in seen]
                s = [cap * math.tanh(a / cap) if cap else a for a in s]
                e = [math.exp(a - slope * (i - j)) for a, j in zip(s, seen)]
                want = sum(a * v[j] for a, j in zip(e, seen)) / sum(e)
                assert torch.allclose(got[i], want, atol=1e-12)
    assert [O.head_slope(h, 4) for h in range(4)] == [0.25, 0.0625, 0.015625, 0.00390625]


def test_oracle_yarn_closed_forms():
    # a factor of 1 changes nothing; without scaling nothing either
    plain, amp = O.yarn(16, 100.0, None)
    same, amp1 = O.yarn(16, 100.0, {"factor": 1.0, "original": 64, "fast": 8.0, "slow": 1.0})
    assert amp == amp1 == 1.0 and all(abs(a - b) < 1e-15 for a, b in zip(plain, same))
    # entry i makes original f_i / (2 pi) turns over the original context: many turns keep their frequency, few are divided
    f, amp = O.yarn(64, 10000.0, {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0})
    base, _ = O.yarn(64, 10000.0, None)
    assert abs(amp - (0.1 * math.log(8.0) + 1.0)) < 1e-15
    for a, b in zip(f, base):
        turns = 4096 * b / (2 * math.pi)
        assert b / 8.0 - 1e-15 <= a <= b + 1e-15
        if turns > 45:
            assert a == b
        if turns < 0.75:
            assert abs(a - b / 8.0) < 1e-15
    assert base[15] > f[15] > base[15] / 8.0
    # rotation: scores depend on the distance only, lengths grow by the amplitude
    g = torch.Generator().manual_seed(2)
    x, y = (torch.randn(1, 1, 8, generator=g, dtype=F64).expand(20, 1, 8).contiguous() for _ in range(2))
    a, b = (O.rotate_half(t, 6, [1.0, 0.3, 0.01], 1.25)[:, 0] for t in (x, y))
    assert torch.allclose(a[:, :6].norm(dim=1), 1.25 * x[:, 0, :6].norm(dim=1)) and torch.equal(a[:, 6:], x[:, 0, 6:])
    assert torch.allclose(a[5] @ b[3], a[17] @ b[15]) and not torch.allclose(a[5] @ b[3], a[17] @ b[14])
    assert abs(float(a[1, 0]) - 1.25 * float(x[0, 0, 0] * math.cos(1.0) - x[0, 0, 3] * math.sin(1.0))) < 1e-12


def test_oracle_streams_and_runs():
    g = torch.Generator().manual_seed(3)
    xs, y, mix, b = torch.randn(5, 3, 4, generator=g, dtype=F64), torch.randn(5, 4, generator=g, dtype=F64), torch.randn(3, 3, generator=g, dtype=F64), torch.randn(3, generator=g, dtype=F64)
    assert torch.allclose(O.write_streams(xs, y, mix, b), torch.einsum("tsw,su->tuw", xs, mix) + b[None, :, None] * y[:, None])
    assert torch.allclose(O.read_streams(xs, b), torch.einsum("tsw,s->tw", xs, b))
    assert O.layer_runs(5, None) == [0, 1, 2, 3, 4] and O.layer_runs(5, {"start": 1, "stop": 3, "times": 3}) == [0, 1, 2, 1, 2, 1, 2, 3, 4]
    # one stream with a mixing matrix of 1 and weights of 1 is an ordinary residual stack
    cfg = U.make_config([(U.attention(), U.moe())], streams=1)
    w = U.make_weights(cfg, 4)
    for q in (1, 2):
        for n in ("in", "out", "mix"):
            w[f"l0.hc{q}.{n}"] = torch.ones_like(w[f"l0.hc{q}.{n}"])
    toks = [3, 9, 7, 7, 1]
    _, layers = O.forward(cfg, w, toks, F64, return_layers=True)
    d = {k: v.to(F64) if v.is_floating_point() else v for k, v in w.items()}
    x = d["embed"][toks]
    x = x + O.attention(O.unit_rms(x, cfg["norm"]["eps"]) * d["l0.norm1"], d, "l0.mix.", cfg["layers"][0]["mixer"])
    x = x + O.table_experts(O.unit_rms(x, cfg["norm"]["eps"]) * d["l0.norm2"], toks, d, "l0.mlp.", cfg["layers"][0]["mlp"])
    assert torch.allclose(layers[0], x, atol=1e-12)


def test_frequencies_of_the_product_follow_the_oracle():
    from llm_quest_amd import kernels_seq as S

    for dims, base, sc in ((64, 1e4, (8.0, 4096, 32.0, 1.0)), (16, 40.0, (4.0, 64, 8.0, 1.0)), (6, 3.0, (2.0, 10, 100.0, 0.01)), (10, 1e6, (1.0, 512, 2.0, 2.0)), (2, 50.0, (40.0, 99, 7.0, 0.1)),
                           (32, 1e3, (16.0, 6, 32.0, 1.0)), (128, 5e5, (4.0, 8192, 32.0, 1.0))):
        scaling = dict(zip(("factor", "original", "fast", "slow"), sc))
        want, amp = O.yarn(dims, base, scaling)
        got, a = S.yarn_rope_frequencies(dims, base, scaling, "cpu")
        assert a == amp and torch.allclose(got.double(), torch.tensor(want, dtype=F64), rtol=1e-7), (dims, base, sc)


def test_config_and_loader_fuse_the_checkpoint():
    from llm_quest_amd.common.mixers import SlidingWindowAttention, TableMoE
    from llm_quest_amd.pavisun.pavisun_model import PavisunConfig, PavisunModel
    from llm_quest_amd.pavisun.pavisun_weight_loading import load_pavisun_state

    cfg = U.make_config(U.default_layers(), loop=(1, 4, 3))
    w = U.make_weights(cfg, 2)
    model = load_pavisun_state(PavisunModel(PavisunConfig(cfg), torch.float32), w)
    assert model.cfg.runs == [0, 1, 2, 3, 1, 2, 3, 1, 2, 3, 4]
    a, b = model.blocks[0].mixer, model.blocks[1].mixer
    assert isinstance(a, SlidingWindowAttention) and a.tie_values and a.slopes is None and not a.gate and a.rot_layout == 1 and (a.window, a.keep_first, a.softcap) == (13, 0, 6.0)
    assert torch.equal(a.w_qkv, torch.cat([w["l0.mix.q"], w["l0.mix.k"]])) and a.b_qkv is None and a.q_norm is None and not a.unit_norm
    assert b.unit_norm and b.gate and not b.tie_values and b.rot_dims == 0 and b.slopes == [O.head_slope(h, 6) for h in range(6)] and (b.window, b.keep_first) == (11, 5)
    assert torch.equal(b.w_qkv, torch.cat([w["l1.mix." + s] for s in ("q", "k", "v", "g")]))
    ff = model.blocks[1].ff
    assert isinstance(ff, TableMoE) and (ff.experts, ff.top, ff.ff) == (5, 3, 24) and torch.equal(ff.table, w["l1.mlp.table"]) and torch.equal(ff.w_down[4], w["l1.mlp.e4.down"])
    assert torch.equal(ff.w_gate_up[2][:24], w["l1.mlp.e2.gate"]) and torch.equal(ff.w_gate_up[2][32:56], w["l1.mlp.e2.up"])
    assert model.blocks[2].ff is None and torch.equal(model.blocks[3].hc2.mix, w["l3.hc2.mix"]) and torch.equal(model.blocks[2].hc1.put, w["l2.hc1.out"])
    cache = model.new_cache("cpu", max_tokens=8, slots=2)
    assert len(cache.layer_specs) == 11  # every pass of a looped layer has rows of its own
    assert cache.rows[0].shape == (2, 8, 2 * 48) and cache.rows[4].shape == cache.rows[1].shape == (2, 8, 2 * 56) and cache.rows[4].data_ptr() != cache.rows[1].data_ptr()


def test_what_the_design_does_not_have_is_refused():
    from llm_quest_amd.common.mixers import SlidingWindowAttention, TableMoE
    from llm_quest_amd.pavisun.pavisun_model import PavisunConfig, PavisunModel

    cfg = U.make_config(U.default_layers())
    PavisunConfig(cfg)
    bad = [{**cfg, "architecture": "Foderax"}, {**cfg, "layers": [{**cfg["layers"][0], "type": "wkv"}]}, {**cfg, "layers": [{**cfg["layers"][0], "mlp": {"kind": "dense", "ff": 8}}]},
           {**cfg, "streams": 0}, {**cfg, "loop": {"start": 2, "stop": 9, "times": 2}}, {**cfg, "loop": {"start": 3, "stop": 2, "times": 2}}, {**cfg, "loop": {"start": 0, "stop": 2, "times": 0}}]
    for c in bad:
        with pytest.raises(ValueError):
            PavisunConfig(c)
    odd = U.make_config([(U.attention(dim=24), None)])
    odd["layers"][0]["mixer"]["vdim"] = 16  # values that are the keys are as wide as they
    with pytest.raises(ValueError):
        PavisunModel(PavisunConfig(odd))
    args = (32, 4, 2, 8, 8, 0.3, 4, 0, 0, 1e4, 1e-5, 0)
    for kw in (dict(slopes=[0.1] * 3), dict(slopes=[0.1] * 4, sigmoid=True), dict(gate=True, head_gate=True), dict(tie_values=True, v_mix="first"), dict(qk_norm="rms"), dict(slopes=[0.1] * 4, pool=2)):
        with pytest.raises(ValueError):
            SlidingWindowAttention(*args, **kw)
    ff = TableMoE(16, 8, 4, 2, 5)
    ff.load_table(torch.tensor([[0, 1], [3, 2], [1, 0], [2, 3], [0, 3]], dtype=torch.int32))
    for t in ([[0, 1]] * 4, [[0, 4]] * 5, [[-1, 0]] * 5, [[2, 2]] * 5):
        with pytest.raises(ValueError):
            ff.load_table(torch.tensor(t, dtype=torch.int32))
    with pytest.raises(ValueError):
        TableMoE(16, 8, 4, 5, 5)


def test_registry_knows_the_design():
    from llm_quest_amd import registry

    assert "Pavisun" in registry.architectures()


def test_serving_bench_configuration_parses_beside_its_reference():
    """The bench's Pavisun model stands beside Mepatar attention layers of about as many weights at both sizes."""
    from llm_quest_amd import serve_bench as B
    from llm_quest_amd.mepatar.mepatar_model import MepatarConfig, MepatarModel
    from llm_quest_amd.pavisun.pavisun_model import PavisunConfig, PavisunModel

    for width, heads in ((1024, 8), (2048, 16)):
        cfg, ref = PavisunConfig(B.pavisun_config(width, heads)), MepatarConfig(B.mepatar_attention_moe_config(width, heads))
        assert len(ref.layers) == len(cfg.runs) == 4 and ref.width == cfg.width
        with torch.device("meta"):
            a = sum(p.numel() for p in PavisunModel(cfg).parameters())
            b = sum(p.numel() for p in MepatarModel(ref).parameters())
        assert 0.97 < a / b < 1.03


def test_the_test_checkpoint_tells_mistakes_apart(monkeypatch):
    """Mistakes planted in the oracle, one at a time, move the logits of the tests' checkpoint by far more than the tolerance of the fp32 tests."""
    cfg = U.make_config(U.default_layers(), loop=(1, 3, 2))
    w = U.make_weights(cfg, 11)
    g = torch.Generator().manual_seed(1)
    toks = torch.randint(0, cfg["vocab"], (70,), generator=g).tolist()
    want = O.forward(cfg, w, toks, F64)
    vis, softmax_head, yarn, write, rms = O.visible, O.softmax_head, O.yarn, O.write_streams, O.unit_rms

    def rotated_values(h, w_, p, m):
        def head(q, k, v, *a):
            return softmax_head(q, k, k, *a)

        monkeypatch.setattr(O, "softmax_head", head)
        try:
            return attention(h, w_, p, m)
        finally:
            monkeypatch.setattr(O, "softmax_head", softmax_head)

    attention = O.attention
    mistakes = {
        "window one longer": ("visible", lambda T, s, k=0: vis(T, s + 1, k)),
        "window one shorter": ("visible", lambda T, s, k=0: vis(T, s - 1, k)),
        "one more token kept": ("visible", lambda T, s, k=0: vis(T, s, k + 1 if k else 0)),
        "one token fewer kept": ("visible", lambda T, s, k=0: vis(T, s, k - 1 if k else 0)),
        "no amplitude": ("yarn", lambda *a: (yarn(*a)[0], 1.0)),
        "unscaled frequencies": ("yarn", lambda d, b, s: (yarn(d, b, None)[0], yarn(d, b, s)[1])),
        "values rotated": ("attention", rotated_values),
        "no cap": ("softmax_head", lambda q, k, v, sc, ok, softcap=0.0, slope=0.0: softmax_head(q, k, v, sc, ok, 0.0, slope)),
        "no distance bias": ("head_slope", lambda h, n: 0.0),
        "slopes from head 0": ("head_slope", lambda h, n: 2.0 ** (-8.0 * h / n)),
        "mixing matrix transposed": ("write_streams", lambda xs, y, m, b: write(xs, y, m.T, b)),
        "one pass of the loop": ("layer_runs", lambda n, loop: list(range(n))),
        "another eps in the head norm": ("unit_rms", lambda x, eps: rms(x, 0.1 if x.dim() == 3 else eps)),
    }
    for name, (attr, repl) in mistakes.items():
        with monkeypatch.context() as mp:
            mp.setattr(O, attr, repl)
            got = O.forward(cfg, w, toks, F64)
        d = got - want
        d = d - d.mean(-1, keepdim=True)
        err = float((d.pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()).max())
        assert err > 0.05, (name, err)
