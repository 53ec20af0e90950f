"""Kaditar without a GPU: the configuration reader, the plan's tensor names, schedule and cache needs, and the plain
implementation against itself (a prompt whole, in portions and token by token), against library routines and against
hand-made cases of its norm, rotation, window, difference of maps, router and copies of the stream."""

import math
import random

import pytest
import torch
import torch.nn.functional as F

from kaditar_cases import CASES, attention, config, dense, double, moe, random_config, tensors_for, with_mlp
from plain import kaditar_plain as P


def build(cfg, dtype=torch.float32):
    from dryft_amd.config.kaditar import KaditarConfig
    from dryft_amd.engine.model import DecoderModel
    from dryft_amd.models import resolve_architecture
    arch = resolve_architecture(cfg)
    assert arch.config_class is KaditarConfig
    return DecoderModel(arch.plan(arch.config_class.from_dict(cfg)), dtype, "cpu")


def check_names(cfg, seed):
    specs = {s.name: tuple(s.shape) for s in build(cfg).tensor_specs()}
    assert specs == {n: tuple(t.shape) for n, t in tensors_for(cfg, seed).items()}


@pytest.mark.parametrize("name", sorted(CASES))
def test_plan_names_every_tensor(name):
    check_names(CASES[name], 1)


def test_random_configurations_are_read():
    for seed in range(40):
        cfg = random_config(random.Random(seed))
        check_names(cfg, seed)
        model = build(cfg)
        assert [r.layer for r in model.plan.schedule] == P.order(cfg)


def test_cache_needs_and_the_loop():
    from dryft_amd.cache.spec import KVNeed
    model = build(CASES["A"], torch.bfloat16)
    runs = model.plan.schedule
    assert [(r.layer, r.cache_line, r.writes_cache, r.enter) for r in runs] == [(l, i, True, None) for i, l in enumerate([0, 1, 2, 1, 2, 3])]
    needs = model.cache_needs()
    assert needs[0] == KVNeed(2, 32, 20) and needs[1] == needs[3] == KVNeed(2, 48, 65) and needs[5] == KVNeed(1, 64, 64)
    # bfloat16 pages hold two maps of a width in steps of 8 and the values, in steps of 16; float32 ones what there is
    b = build(CASES["B"], torch.bfloat16).cache_needs()
    assert b[0] == KVNeed(3, 48, None) and b[1] == KVNeed(2, 64, 9)
    f = build(CASES["B"]).cache_needs()
    assert f[0] == KVNeed(3, 40, None, 12) and f[1] == KVNeed(2, 26, 9, 50) and len(f) == 6
    c = build(CASES["C"], torch.bfloat16).cache_needs()
    assert c[2] == KVNeed(1, 272, 70, 40)                             # beyond the matrix-core kernels: as float32 does
    assert c[3] == KVNeed(2, 208, None)


def test_configuration_problems_come_in_one_error():
    from dryft_amd.config.base import ConfigError
    from dryft_amd.config.kaditar import KaditarConfig
    bad = config(64, 100, 9, [with_mlp(attention(3, 2, 16, 16, rot=20), moe(4, 5, 8)), attention(2, 1, 300, 16),
                              {"type": "wkv", "mixer": {}}, with_mlp(attention(2, 2, 8, 8), {"kind": "glu"})], loop=(2, 9, 2))
    del bad["layers"][1]["mixer"]["diff"]
    bad["layers"][3]["mixer"]["mask"] = {"size": 0}
    bad["logit_softcap"] = -1.0
    with pytest.raises(ConfigError) as e:
        KaditarConfig.from_dict(bad)
    text = "\n".join(e.value.problems)
    for piece in ("streams: at most", "logit_softcap: must be > 0", "layers[0].mixer.heads (3) is not a multiple",
                  "layers[0].mixer.rot.dims", "layers[0].mlp.router.top", "layers[1].mixer.diff: missing",
                  "layers[1].mixer.dim, vdim", "layers[2]: expected", "layers[3].mixer.mask.size", "layers[3].mlp.kind",
                  "loop: start 2 .. stop 9"):
        assert piece in text, piece


def test_configuration_writes_back_what_it_read():
    from dryft_amd.config.kaditar import KaditarConfig
    import dataclasses
    for cfg in CASES.values():
        read = KaditarConfig.from_dict(cfg)
        assert read.to_dict() == cfg
        again = KaditarConfig.from_dict(dataclasses.replace(read, raw=()).to_dict())
        assert dataclasses.replace(again, raw=()) == dataclasses.replace(read, raw=())


def test_layer_order():
    from dryft_amd.config.base import LoopConfig, layer_order
    assert layer_order(3, None) == [(0, None), (1, None), (2, None)]
    assert layer_order(4, LoopConfig(1, 3, 2)) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert layer_order(2, LoopConfig(0, 1, 3)) == [(0, 0), (0, 1), (0, 2), (1, None)]


def test_the_maps_factor_is_one_number_of_the_layer():
    from dryft_amd.parts.diff_attention import DifferentialAttention
    g = torch.Generator().manual_seed(0)
    part = DifferentialAttention(24, 2, 1, 6, 12, 0.4, 0.3, 1e-5)
    t = {n: torch.randn(s, generator=g) for n, (s, _, _) in part.tensor_specs().items()}
    part.load(t)
    want = math.exp(float((t["lq1"] * t["lk1"]).sum())) - math.exp(float((t["lq2"] * t["lk2"]).sum())) + 0.3
    assert part.lam == pytest.approx(want, rel=1e-6)
    assert float(P.difference(double(t), {"diff": 0.3})) == pytest.approx(want, rel=1e-6)


# ------------------------------------------------------------------------------------------ plain against library routines
def test_layer_norm_against_torch():
    g = torch.Generator().manual_seed(0)
    x = 5 + 3 * torch.randn(7, 40, generator=g, dtype=torch.float64)
    w, b = torch.randn(2, 40, generator=g, dtype=torch.float64)
    assert torch.allclose(P.layer_norm(x, w, b, 1e-3), F.layer_norm(x, (40,), w, b, 1e-3), atol=1e-12)
    one = torch.tensor([[1.0, 3.0]], dtype=torch.float64)                 # mean 2, variance 1
    assert torch.allclose(P.layer_norm(one, 1.0, 0.5, 3.0), torch.tensor([[0.0, 1.0]], dtype=torch.float64))


def test_attention_against_torch():
    """Without the difference's norm, a head is the difference of two library attentions over the same values."""
    g = torch.Generator().manual_seed(1)
    c = {"heads": 4, "kv_heads": 2, "dim": 8, "vdim": 6, "scale": 0.3, "diff": 0.4, "mask": {"size": 3}}
    w = {n: torch.randn(r, 10, generator=g, dtype=torch.float64) for n, r in (("q", 64), ("k", 32), ("v", 12))}
    w.update({n + ".b": torch.randn(r, generator=g, dtype=torch.float64) for n, r in (("q", 64), ("k", 32), ("v", 12))})
    w.update({n: 0.3 * torch.randn(8, generator=g, dtype=torch.float64) for n in ("lq1", "lk1", "lq2", "lk2")})
    w["o"] = torch.eye(24, dtype=torch.float64)
    h = torch.randn(9, 10, generator=g, dtype=torch.float64)
    lam = math.exp(float(w["lq1"] @ w["lk1"])) - math.exp(float(w["lq2"] @ w["lk2"])) + 0.4
    q, k, v = (F.linear(h, w[n], w[n + ".b"]) for n in "qkv")
    i, j = torch.arange(9)[:, None], torch.arange(9)[None]
    mask = (j <= i) & (j > i - 3)
    want = []
    for head in range(4):
        kv = head // 2
        a = [F.scaled_dot_product_attention(q[:, 16 * head + 8 * m:][:, :8][None], k[:, 16 * kv + 8 * m:][:, :8][None],
                                            v[:, 6 * kv:][:, :6][None], attn_mask=mask, scale=0.3)[0] for m in (0, 1)]
        want.append(F.rms_norm(a[0] - lam * a[1], (6,), None, 1e-5) * 0.6)
    got, past = P.attention(h, w, c, 1e-5)
    assert torch.allclose(got, torch.cat(want, -1), atol=1e-12)
    assert past[0].shape == (9, 2, 2, 8) and past[1].shape == (9, 2, 6)


def test_the_window_counts_the_row_itself():
    seen = P.visible(torch.arange(5, 7), torch.arange(8), 3)
    assert seen.tolist() == [[False] * 3 + [True] * 3 + [False] * 2, [False] * 4 + [True] * 3 + [False]]
    assert P.visible(torch.arange(2, 3), torch.arange(4), None).tolist() == [[True] * 3 + [False]]


def test_rotation_by_hand():
    x = torch.tensor([[[1.0, 0.0, 0.0, 2.0, 5.0]]], dtype=torch.float64)
    a0, a1 = 3.0, 3.0 * 100.0 ** -0.5
    want = [math.cos(a0), math.sin(a0), -2 * math.sin(a1), 2 * math.cos(a1), 5.0]
    got = P.rotate_pairs(x, torch.tensor([3]), {"dims": 4, "base": 100.0})
    assert torch.allclose(got[0, 0], torch.tensor(want, dtype=torch.float64), atol=1e-12)
    assert P.rotate_pairs(x, torch.tensor([3]), None) is x


def test_router_by_hand():
    w = {"router": torch.eye(4, dtype=torch.float64), "router.b": torch.tensor([0.0, 0.0, 2.0, 0.0], dtype=torch.float64)}
    chosen, weights = P.route(torch.tensor([[1.0, 0.5, -0.5, 0.0]], dtype=torch.float64), w, {"router": {"top": 2}})
    assert chosen.tolist() == [[2, 0]]                                    # the bias decides, and weighs too
    e = math.exp(1.5), math.exp(1.0)
    assert torch.allclose(weights[0], torch.tensor([e[0] / sum(e), e[1] / sum(e)], dtype=torch.float64))


def test_copies_are_mixed_from_to():
    streams = [torch.tensor([1.0]), torch.tensor([10.0])]
    hc = {"mix": torch.tensor([[1.0, 2.0], [3.0, 4.0]]), "out": torch.tensor([100.0, 1000.0])}
    assert [float(x) for x in P.mixed_streams(streams, hc, torch.tensor([1.0]))] == [131.0, 1042.0]


def test_capped_logits():
    z = torch.tensor([-1e4, 0.5, 1e4], dtype=torch.float64)
    assert torch.allclose(P.capped(z, 15.0), torch.tensor([-15.0, 15 * math.tanh(0.5 / 15), 15.0], dtype=torch.float64))
    assert P.capped(z, None) is z


# ------------------------------------------------------------------------------------------ plain against itself
@pytest.mark.parametrize("name", sorted(CASES))
def test_plain_whole_in_portions_and_token_by_token(name):
    cfg = CASES[name]
    t = double(tensors_for(cfg, 3))
    toks = torch.randint(0, cfg["vocab"], (150,), generator=torch.Generator().manual_seed(5)).tolist()
    taps = []
    whole, _ = P.forward(cfg, t, toks, taps=taps)
    assert len(taps) == len(P.order(cfg)) and taps[0].shape == (150, cfg["width"])
    for cuts in ([2, 4, 64, 66, 129], list(range(120, 150))):
        past, rows = None, []
        edges = [0] + cuts + [150]
        for a, b in zip(edges[:-1], edges[1:]):
            out, past = P.forward(cfg, t, toks[a:b], past)
            rows.append(out)
        assert torch.allclose(torch.cat(rows), whole, atol=1e-8), cuts[:3]


def test_a_pass_has_a_cache_of_its_own():
    """Were the passes to share keys and values, a model of one looped layer would see its first pass's rows twice."""
    cfg = config(32, 50, 2, [with_mlp(attention(2, 1, 8, 16, rot=4), dense(24))], loop=(0, 1, 2))
    t = double(tensors_for(cfg, 5))
    toks = list(range(20))
    want, state = P.forward(cfg, t, toks)
    assert len(state) == 2 and not torch.allclose(state[0][0], state[1][0], atol=1e-2)
    swapped = [state[1], state[0]]
    a, b = P.forward(cfg, t, [7], state)[0], P.forward(cfg, t, [7], swapped)[0]
    assert float((a - b).abs().max()) > 1e-2
