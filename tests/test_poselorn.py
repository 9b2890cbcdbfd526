"""Poselorn without a GPU: the reader of ``config.json``, the layout it gives, the plain mechanisms on hand-made cases, and
the new kernels' plain twins against the plain mechanisms."""

from __future__ import annotations

import copy
import math

import pytest
import torch

from fastgen_amd.config import ConfigError, PartSpec, get_architecture
from fastgen_amd.engine.model import build_parts
from fastgen_amd.kernels import ops, twins
from fastgen_amd.parts import build_part
from plain_poselorn import (ODD, ONLY_DELTA, ONLY_LEFT, QUARTET, WIDE, plain_channel_delta, plain_conv, plain_decayed_attention,
                            plain_dense, plain_experts, plain_forward, plain_order, plain_rms, plain_rotate, plain_route, plain_silu,
                            plain_unit, plain_weights, plain_window, plain_window_attention)

ALL = (QUARTET, ODD, WIDE, ONLY_LEFT, ONLY_DELTA)


def _shapes(config, **ranks):
    return {k: tuple(v.shape) for k, v in plain_weights(config, 0, **ranks).items()}


# ------------------------------------------------------------------ reader and layout
def test_the_reader_round_trips_and_names_what_is_wrong():
    arch = get_architecture(QUARTET)
    assert arch.name == "Poselorn"
    for config in ALL:
        args = arch.parse(config, _shapes(config).get)
        assert arch.parse(arch.to_hf_config(args)) == args

    def broken(change, match):
        c = copy.deepcopy(QUARTET)
        change(c)
        with pytest.raises(ConfigError, match=match):
            arch.parse(c)

    left = lambda c: c["layers"][0]["mixer"]["left"]
    right = lambda c: c["layers"][0]["mixer"]["right"]
    router = lambda c: c["layers"][1]["mlp"]["router"]
    broken(lambda c: left(c).pop("vdim"), "vdim")
    broken(lambda c: left(c)["rot"].update(dims=18), "rot.dims")
    broken(lambda c: left(c)["mask"].update(size=0), "window")
    broken(lambda c: right(c).update(decay=[0.5, 0.5]), "decay")
    broken(lambda c: right(c).update(decay=[0.5, 0.5, 1.5]), "decay")
    broken(lambda c: c["layers"][1]["mixer"].update(heads=3), "heads")
    broken(lambda c: c["layers"][1]["mixer"].pop("conv"), "conv")
    broken(lambda c: router(c).update(identity=3), "groups")
    broken(lambda c: router(c)["groups"].update(keep=4), "groups")
    broken(lambda c: router(c).update(top=9), "top")
    broken(lambda c: c["layers"][0]["mlp"].update(kind="glu"), "glu")
    broken(lambda c: c["layers"][0].update(type="rnn"), "rnn")
    broken(lambda c: c["loop"].update(stop=9), "loop")
    broken(lambda c: c.pop("norm"), "norm")


def test_the_layout_names_every_tensor_and_asks_for_pages_and_state():
    arch = get_architecture(QUARTET)
    for config in ALL:
        for ranks in ({}, dict(a_rank=9, g_rank=3)):
            shapes = _shapes(config, **ranks)
            parts = build_parts(arch.layout(arch.parse(config, shapes.get)))
            assert {s.name: tuple(s.shape) for s in parts.tensor_specs()} == shapes
    parts = build_parts(arch.layout(arch.parse(QUARTET)))
    paged = [m.paged_need() for m in parts.mixers]
    assert [p is not None for p in paged] == [True, False, True, False]
    assert (paged[0].n_kv_heads, paged[0].head_dim, paged[0].window) == (2, 32, 20)  # the wider of 16 and 24, in steps of 16
    assert (paged[2].n_kv_heads, paged[2].head_dim, paged[2].window) == (1, 16, 32)
    state = [m.state_need().shape for m in parts.mixers]
    assert state == [(3, 16, 8), (4 * 16 * 24 + (2 * 2 * 16 + 4 * 24) * 2,), (2, 24, 16), (2 * 32 * 16 + (2 * 2 * 32 + 2 * 16),)]
    # the middle layers run three times with storage of their own, and the embedding enters before all passes but the first
    layout = arch.layout(arch.parse(QUARTET))
    assert [(e.layer, e.inject is not None) for e in layout.order] == plain_order(QUARTET) \
        == [(0, False), (1, False), (2, False), (1, True), (2, False), (1, True), (2, False), (3, False)]
    assert all(e.reads_cache_of is None for e in layout.order)
    once = copy.deepcopy(QUARTET)
    once["loop"]["times"] = 1
    assert not arch.layout(arch.parse(once)).injections


def test_options_that_do_not_go_together_are_refused():
    right = PartSpec("lightning_attention", "a", dict(dim=8, n_heads=1, head_dim=8, v_head_dim=8, decay=[0.5], eps=1e-5))
    left = PartSpec("attention", "b", dict(dim=8, n_heads=1, n_kv_heads=1, head_dim=8, position=PartSpec("none"), prepared=True))
    with pytest.raises(ValueError, match="side by side"):
        build_part("mixer", PartSpec("parallel_mixers", "m", dict(dim=8, left=right, right=right)))
    both = build_part("mixer", PartSpec("parallel_mixers", "m", dict(dim=8, left=left, right=right, out_norms=True, eps=1e-5)))
    norm = build_part("norm", PartSpec("rmsnorm", "n", dict(dim=8, eps=1e-5)))
    other = build_part("norm", PartSpec("rmsnorm", "n", dict(dim=8, eps=1e-6)))
    mlp = build_part("feed_forward", PartSpec("mlp", "f", dict(dim=8, hidden_dim=8, bias=True)))
    for kind in ("pre_norm", "parallel", "norm_behind"):
        with pytest.raises(ValueError, match="sum of normed rows"):
            build_part("arrangement", PartSpec(kind), both, None, norm, None if kind == "parallel" else norm)
    scaled = PartSpec("parallel_scaled", "l", dict(dim=8))
    build_part("arrangement", scaled, both, mlp, norm, norm)
    with pytest.raises(ValueError, match="eps"):
        build_part("arrangement", scaled, both, mlp, norm, other)
    with pytest.raises(ValueError, match="decays"):
        build_part("mixer", PartSpec("lightning_attention", "a", dict(right.options, decay=[0.5, 0.5])))
    moe = dict(dim=8, hidden_dim=8, n_experts=4, top=2, router_bias=False)
    with pytest.raises(ValueError, match="raw weights"):
        build_part("feed_forward", PartSpec("moe", "f", dict(moe, renormalize=False)))
    with pytest.raises(ValueError, match="fit"):
        build_part("feed_forward", PartSpec("moe", "f", dict(moe, scoring="softmax_all", identity=1, n_groups=2)))
    with pytest.raises(ValueError, match="group_rank"):
        build_part("feed_forward", PartSpec("moe", "f", dict(moe, scoring="softmax_all", group_rank="sum")))


# ------------------------------------------------------------------ plain mechanisms by hand
def test_window_and_rotation_by_hand():
    assert plain_window(5, 2)[3].tolist() == [False, False, True, True, False]
    q = torch.zeros(4, 1, 2)
    v = torch.tensor([[[1.0]], [[2.0]], [[4.0]], [[9.0]]])
    o = plain_window_attention(q, torch.randn(4, 1, 2), v, 1.0, 2)
    assert o.flatten().tolist() == [1.0, 1.5, 3.0, 6.5]
    x = torch.zeros(3, 1, 6)
    x[:, 0, 0], x[:, 0, 5] = 1.0, 7.0  # dimension 0 pairs with dimension 2 of four; 4 and 5 pass
    y = plain_rotate(x, 100.0, 4)
    for p in range(3):
        assert torch.allclose(y[p, 0], torch.tensor([math.cos(p), 0.0, math.sin(p), 0.0, 0.0, 7.0]), atol=1e-6)
    assert plain_conv(torch.tensor([[1.0], [10.0], [100.0]]), torch.tensor([[3.0, 2.0, 1.0]])).flatten().tolist() == [1.0, 12.0, 123.0]


def test_recurrences_by_hand():
    one = torch.ones(3, 1)
    assert plain_decayed_attention(one, one, torch.tensor([[4.0], [2.0], [1.0]]), 0.5).flatten().tolist() == [4.0, 4.0, 3.0]
    # the delta rule with a decay per channel: a second write replaces the first in proportion to beta; channel 1 fades alone
    k = torch.tensor([[1.0, 0.0], [1.0, 0.0], [0.0, 1.0], [1.0, 0.0]])
    v = torch.tensor([[2.0], [6.0], [5.0], [4.0]])
    g = torch.tensor([[1.0, 1.0], [1.0, 1.0], [1.0, 1.0], [1.0, 0.5]])
    o = plain_channel_delta(torch.ones(4, 2), k, v, g, torch.tensor([1.0, 0.5, 1.0, 0.0]))
    assert o.flatten().tolist() == [2.0, 4.0, 4.0 + 5.0, 4.0 + 2.5]
    assert torch.allclose(plain_unit(torch.tensor([3.0, 4.0])), torch.tensor([0.6, 0.8]), atol=1e-6)


def test_feed_forwards_by_hand():
    w = {"f.up": torch.tensor([[2.0], [-1.0]]), "f.up.b": torch.tensor([1.0, 0.5]), "f.down": torch.tensor([[1.0, 5.0]]),
         "f.down.b": torch.tensor([0.25])}
    assert plain_dense(torch.ones(1, 1), w, "f", torch.float32).tolist() == [[9.25]]
    # scores 0.4, 0.3, 0.2, 0.1; groups of two by their best: the correction makes the second group the better one
    z = torch.log(torch.tensor([0.4, 0.3, 0.2, 0.1]))
    none = torch.zeros(4)
    assert plain_route(z, none, 2, 1, 1)[0] == [0, 1]
    assert plain_route(z, none, 2, 2, 1)[0] == [0, 1]
    chosen, weight = plain_route(z, torch.tensor([0.0, 0.0, 0.0, 0.35]), 2, 2, 1)
    assert chosen == [3, 2] and torch.allclose(torch.tensor(weight), torch.tensor([0.1, 0.2]))
    chosen, _ = plain_route(z, torch.full((4,), -5.0), 2, 2, 1)  # choice scores may be negative: the others are out all the same
    assert chosen == [0, 1]
    # an identity expert returns its input
    w = {"f.router": torch.eye(2), "f.correction": torch.zeros(2), "f.e0.gate": torch.ones(1, 2), "f.e0.up": torch.ones(1, 2),
         "f.e0.down": torch.ones(2, 1)}
    h = torch.tensor([[0.0, 2.0]])
    y = plain_experts(h, w, "f", {"router": {"experts": 1, "identity": 1, "top": 1}}, torch.float32)
    assert torch.allclose(y, torch.softmax(h[0], 0)[1] * h)


def test_every_mechanism_moves_the_logits():
    """The random weights of these tests are large enough that leaving a mechanism out shows."""
    toks = torch.randint(0, QUARTET["vocab"], (50,), generator=torch.Generator().manual_seed(4)).tolist()
    w = plain_weights(QUARTET, 1)
    base = plain_forward(w, QUARTET, toks)
    scale = float(base.abs().max())

    def moved(change_w=None, change_c=None):
        w2, c2 = {k: v.clone() for k, v in w.items()}, copy.deepcopy(QUARTET)
        if change_w:
            change_w(w2)
        if change_c:
            change_c(c2)
        return float((plain_forward(w2, c2, toks) - base).abs().max()) / scale

    for name in ("l0.mix.left.q.b", "l0.mix.left.k.norm", "l0.mix.left.v.b", "l0.mix.left.q.norm", "l0.mix.left.out", "l0.mix.right.out",
                 "l0.mix.right.norm", "l0.mix.right.g", "l1.mix.A_log", "l1.mix.dt_bias", "l1.mix.b", "l1.mix.norm", "l1.mix.a1",
                 "l1.mix.a2", "l1.mix.g1", "l1.mix.g2", "l0.ls1", "l1.ls2", "l1.norm1", "l1.norm2", "l0.mlp.up.b", "l0.mlp.down.b"):
        direction = torch.randn(w[name].shape, generator=torch.Generator().manual_seed(len(name)))
        assert moved(lambda w2: w2[name].add_(0.5 * direction)) > 1e-3, name
    for name in ("l1.mix.q.conv", "l1.mix.k.conv", "l1.mix.v.conv"):
        assert moved(lambda w2: w2[name][:, 0].zero_()) > 1e-3, name
    # a key's bias moves all of a query's scores by one number where nothing is normed or rotated; here it does not
    assert moved(lambda w2: w2["l0.mix.left.k.b"].add_(0.5)) > 1e-3
    assert moved(lambda w2: w2["l1.mlp.correction"].neg_()) > 1e-3
    left = lambda c: c["layers"][0]["mixer"]["left"]
    assert moved(change_c=lambda c: left(c)["mask"].update(size=19)) > 1e-3
    assert moved(change_c=lambda c: left(c)["rot"].update(base=50.0)) > 1e-3
    assert moved(change_c=lambda c: left(c).update(scale=0.4)) > 1e-3
    assert moved(change_c=lambda c: c["layers"][0]["mixer"]["right"].update(decay=[0.5, 0.93, 0.99])) > 1e-3
    assert moved(change_c=lambda c: c["layers"][1]["mlp"]["router"].pop("groups")) > 1e-3
    assert moved(change_c=lambda c: c["layers"][1]["mlp"]["router"].update(top=2)) > 1e-3
    assert moved(change_c=lambda c: c.update(residual_mult=0.5)) > 1e-3
    assert moved(change_c=lambda c: c["embedding"].update(scale=2.0)) > 1e-3
    assert moved(change_c=lambda c: c["loop"].update(times=2)) > 1e-3


# ------------------------------------------------- the kernels' twins against the plain mechanisms
def test_twin_of_the_terms():
    g = torch.Generator().manual_seed(0)
    r = lambda *s: torch.randn(*s, generator=g)
    h, a, b, again, s, t, bias, w1, w2 = r(4, 10), r(4, 10), r(2, 4, 10), r(4, 10), r(10), r(10), r(10), r(10), r(10)
    want = h + plain_rms(a, s, 1e-3) + t * (b.sum(0) + bias)
    terms = ops.StreamTerms([ops.StreamTerm(a, s, None, 1e-3), ops.StreamTerm(b, t, bias)])
    o1, o2 = torch.empty(4, 10), torch.empty(4, 10)
    hh = h.clone()
    twins.stream_terms(hh, terms, None, [(w1, o1), (w2, o2)], 1e-5)
    torch.testing.assert_close(hh, want)
    torch.testing.assert_close(o1, plain_rms(want, w1, 1e-5))
    torch.testing.assert_close(o2, plain_rms(want, w2, 1e-5))
    hh, o1 = h.clone(), torch.empty(2, 10)
    twins.stream_terms(hh, terms, again, [(w1, o1)], 1e-5, torch.tensor([3, 1], dtype=torch.int32))
    assert torch.equal(hh, h)
    torch.testing.assert_close(o1, plain_rms((want + again)[[3, 1]], w1, 1e-5))
    # every form of what a layer leaves to be added is terms
    for delta, add in ((a, a), (b, b.sum(0)), (ops.ScaledDelta(a, s), a * s), (ops.PostNormed(a, s, 1e-3, bias), plain_rms(a + bias, s, 1e-3)),
                       (None, 0.0), (terms, want - h)):
        hh = h.clone()
        twins.stream_terms(hh, ops.StreamTerms.of(delta))
        torch.testing.assert_close(hh, h + add, rtol=1e-5, atol=1e-5)


def test_twins_of_norms_gates_and_activations():
    g = torch.Generator().manual_seed(1)
    x, w, gate, out = torch.randn(3, 12, generator=g), torch.rand(12, generator=g), torch.randn(3, 15, generator=g), torch.zeros(3, 12)
    twins.row_norm_gate(x, w, 1e-5, gate, out, 0.5)
    torch.testing.assert_close(out, 0.5 * plain_rms(x, w, 1e-5) * torch.sigmoid(gate[:, :12]))
    twins.head_norm_gate(x, w[:4], 1e-5, gate, 3, out, sigmoid=True)
    torch.testing.assert_close(out, plain_rms(x.view(3, 3, 4), w[:4], 1e-5).reshape(3, 12) * torch.sigmoid(gate[:, :12]))
    torch.testing.assert_close(twins.bias_act(x, w, "relu2", torch.float32), torch.relu(x + w) ** 2)
    torch.testing.assert_close(twins.bias_act(x, None, "silu", torch.float32), plain_silu(x))
    a, b = torch.zeros(3, 6), torch.zeros(3, 5)
    w2, w3, rate, bias = torch.randn(6, 4, generator=g), torch.randn(5, 3, generator=g), torch.rand(2, generator=g), torch.randn(6, generator=g)
    twins.low_rank(x, [ops.LowRankJob(2, w2, a, bias, rate, 3), ops.LowRankJob(8, w3, b)])
    torch.testing.assert_close(b, x[:, 8:11] @ w3.T)
    step = torch.nn.functional.softplus(x[:, 2:6] @ w2.T + bias)
    torch.testing.assert_close(a, -step * rate[[0, 0, 0, 1, 1, 1]])


def test_twins_of_the_router_with_identity_experts():
    g = torch.Generator().manual_seed(2)
    T, D, E, I, top = 9, 8, 5, 3, 3
    x, router, corr = torch.randn(T, D, generator=g), torch.randn(E + I, D, generator=g), 0.2 * torch.randn(E + I, generator=g) - 0.3
    choice, weight = twins.moe_route(x, router, None, top, softmax_scores=True, correction=corr, n_groups=4, keep_groups=2,
                                     group_max=True, raw_weights=True)
    for t in range(T):
        chosen, w = plain_route(router @ x[t], corr, top, 4, 2)
        assert choice[t].tolist() == chosen
        torch.testing.assert_close(weight[t], torch.tensor(w))
    sorted_, tiles = twins.moe_sort(choice, E + I, 16, I)
    assert sorted(sorted_.tolist()) == list(range(T * top)) and all(e < E for e, _, n, _ in tiles.tolist() if n)
    assert sum(n for _, _, n, _ in tiles.tolist()) == int((choice < E).sum())
    y = torch.randn(T * top, D, generator=g)
    y[(choice.reshape(-1) >= E)] = float("nan")
    got = twins.moe_combine(y, weight, None, None, choice, E, x)[0]
    want = torch.stack([sum(weight[t, j] * (x[t] if choice[t, j] >= E else y[t * top + j]) for j in range(top)) for t in range(T)])
    torch.testing.assert_close(got, want)


def test_twins_of_the_recurrences():
    G, d, H, e, K = 2, 6, 4, 8, 3
    C, lens = 2 * G * d + H * e, [7, 1, 4]
    T = sum(lens)
    g = torch.Generator().manual_seed(9)
    q_start = torch.tensor([0, 7, 8, 12], dtype=torch.int32)
    slots = torch.tensor([4, 0, 3], dtype=torch.int32)
    seq = torch.repeat_interleave(torch.arange(3), torch.tensor(lens)).to(torch.int32)
    conv = ops.ConvInputs(torch.randn(C, K, generator=g), torch.zeros(6, C, K - 1), 0, slots, seq, q_start, False)
    src = torch.randn(T, C + H, generator=g)
    ready = torch.zeros(T, C + H + 2 + H * d)
    twins.delta_prepare(src, G, d, H, e, conv, C, -1, None, None, d ** -0.5, 1e-6, ready)
    ready[:, C + H + 2 :] = log_g = -torch.rand(T, H * d, generator=g)
    state, out = torch.zeros(6, H, d, e), torch.empty(T, H * e)
    twins.delta_scan(ready, G, d, H, e, state, slots, q_start, 3, out, None, C + H + 2)
    rows = torch.randn(T, 2 * H * d + H * e, generator=g)
    decay = torch.tensor([0.2, 0.9, 1.0, 0.99])
    s2, o2 = torch.zeros(6, H, d, e), torch.empty(T, H * e)
    twins.lightning_scan(rows, 0, H * d, 2 * H * d, torch.log(decay), s2, slots, q_start, 3, o2)
    for b, n in enumerate(lens):
        at = slice(int(q_start[b]), int(q_start[b + 1]))
        y = plain_silu(plain_conv(src[at, :C], conv.taps))
        q, k = plain_unit(y[:, : G * d].view(n, G, d)) * d ** -0.5, plain_unit(y[:, G * d : 2 * G * d].view(n, G, d))
        v, beta, gg = y[:, 2 * G * d :].view(n, H, e), torch.sigmoid(src[at, C : C + H]), torch.exp(log_g[at]).view(n, H, d)
        want = torch.stack([plain_channel_delta(q[:, h // 2], k[:, h // 2], v[:, h], gg[:, h], beta[:, h]) for h in range(H)], 1)
        torch.testing.assert_close(out[at], want.reshape(n, -1), rtol=1e-5, atol=1e-5)
        z = plain_silu(rows[at])
        q, k, v = (z[:, c : c + H * w].view(n, H, w) for c, w in ((0, d), (H * d, d), (2 * H * d, e)))
        want = torch.stack([plain_decayed_attention(q[:, h], k[:, h], v[:, h], float(decay[h])) for h in range(H)], 1)
        torch.testing.assert_close(o2[at], want.reshape(n, -1), rtol=1e-5, atol=1e-5)


def test_a_whole_model_in_float64_and_float32_agree():
    for config in (QUARTET, ODD, WIDE):
        w = plain_weights(config, 3)
        toks = [t % config["vocab"] for t in range(5, 45)]
        a, b = plain_forward(w, config, toks, torch.float64), plain_forward(w, config, toks)
        assert float((a - b.double()).abs().max()) < 1e-4 * float(a.abs().max())
