"""Ropelix without a GPU: the reader of ``config.json``, the layout it gives, the plain mechanisms on hand-made cases,
and the new kernels' plain twins against the plain mechanisms."""

from __future__ import annotations

import copy
import math

import pytest
import torch

from fastgen_amd.cache.layout import pack_k, pack_v
from fastgen_amd.config import ConfigError, get_architecture
from fastgen_amd.engine.model import build_parts
from fastgen_amd.kernels import ops, twins
from plain_ropelix import (ODD, ONLY_CONV, ONLY_DELTA, ONLY_MIXED, TRIO, WIDE, plain_block_linear, plain_conv,
                           plain_delta_rule, plain_distance_bias, plain_feed_forward, plain_forward, plain_gelu,
                           plain_heads_attend, plain_lru, plain_mix_heads, plain_rms, plain_rotate, plain_scores, plain_silu,
                           plain_softcap, plain_unit, plain_weights, plain_weights_of, plain_window)


# ------------------------------------------------------------------ reader and layout
def test_the_reader_round_trips_and_names_what_is_wrong():
    arch = get_architecture(TRIO)
    assert arch.name == "Ropelix"
    for config in (TRIO, ODD, WIDE, ONLY_MIXED, ONLY_CONV, ONLY_DELTA):
        args = arch.parse(config)
        assert arch.parse(arch.to_hf_config(args)) == args

    def broken(change, match):
        c = copy.deepcopy(TRIO)
        change(c)
        with pytest.raises(ConfigError, match=match):
            arch.parse(c)

    broken(lambda c: c["layers"][0]["mixer"]["left"].pop("vdim"), "vdim")
    broken(lambda c: c["layers"][0]["mixer"]["right"].update(blocks=5), "blocks")
    broken(lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=18), "rot.dims")
    broken(lambda c: c["layers"][1]["mixer"].update(heads=3), "heads")
    broken(lambda c: c["layers"][2]["mixer"].update(vdim=8), "vdim")
    broken(lambda c: c["layers"][2]["mixer"]["mask"].update(size=0), "window")
    broken(lambda c: c["layers"][0]["mlp"].update(kind="moe"), "kind")
    broken(lambda c: c["layers"][0].update(type="rnn"), "rnn")
    broken(lambda c: c.pop("norm"), "norm")


def test_the_layout_names_every_tensor_and_asks_for_pages_and_state():
    arch = get_architecture(TRIO)
    for config in (TRIO, ODD, WIDE):
        parts = build_parts(arch.layout(arch.parse(config)))
        assert {s.name: tuple(s.shape) for s in parts.tensor_specs()} == {k: tuple(v.shape) for k, v in plain_weights(config, 0).items()}
    parts = build_parts(arch.layout(arch.parse(TRIO)))
    paged = [m.paged_need() for m in parts.mixers]
    assert [p is not None for p in paged] == [True, False, True, False]
    assert (paged[0].n_kv_heads, paged[0].head_dim, paged[0].window) == (2, 32, 20)  # the wider of 16 and 24, in steps of 16
    assert (paged[2].n_kv_heads, paged[2].head_dim, paged[2].window) == (2, 16, 23)
    state = [m.state_need().shape for m in parts.mixers]
    assert state == [(48, 4), (4 * 16 * 24 + (2 * 2 * 16 + 4 * 24) * 2,), ((4 + 2) * 16, 1), (3 * 32 * 16 + (2 * 3 * 32 + 3 * 16),)]


def test_options_that_do_not_go_together_are_refused():
    from fastgen_amd.config import PartSpec
    from fastgen_amd.parts import build_part

    with pytest.raises(ValueError, match="side by side"):
        side = PartSpec("gated_linear_recurrence", "a", dict(dim=8, width=8, blocks=2, taps=2))
        build_part("mixer", PartSpec("parallel_mixers", "m", dict(dim=8, left=side, right=side)))
    with pytest.raises(ValueError, match="value_from_key"):
        build_part("mixer", PartSpec("attention", "a", dict(
            dim=8, n_heads=2, n_kv_heads=1, head_dim=8, conv_taps=2, value_from_key=True,
            position=PartSpec("rope", options=dict(head_dim=8, theta=10.0)))))
    with pytest.raises(ValueError, match="exact"):
        build_part("mixer", PartSpec("attention", "a", dict(dim=8, n_heads=2, n_kv_heads=1, head_dim=8, distance_bias=True,
                                                            position=PartSpec("none"))))
    with pytest.raises(ValueError, match="blocks"):
        build_part("mixer", PartSpec("gated_linear_recurrence", "a", dict(dim=8, width=10, blocks=4, taps=2)))


# ------------------------------------------------------------------ plain mechanisms by hand
def test_window_softcap_sink_and_mixing_by_hand():
    assert plain_window(5, 2)[3].tolist() == [False, False, True, True, False]
    assert plain_window(3, None)[2].tolist() == [True, True, True]
    assert torch.allclose(plain_softcap(torch.tensor([1e9, -1e9, 0.0]), 4.0), torch.tensor([4.0, -4.0, 0.0]))
    s = torch.tensor([[[0.0, 0.0], [math.log(2.0), 0.0]]])
    a = plain_weights_of(s, plain_window(2, None), plus_one=True)
    assert torch.allclose(a[0, 1], torch.tensor([0.5, 0.25]))  # 2 : 1 : 1
    assert torch.allclose(plain_weights_of(s, plain_window(2, 1))[0, 1], torch.tensor([0.0, 1.0]))
    w = torch.tensor([[[1.0, 0.0]], [[0.25, 0.75]]])
    mixed = plain_mix_heads(w, torch.tensor([[2.0, 0.0], [1.0, -1.0]]))
    assert torch.allclose(mixed[0, 0], torch.tensor([2.0, 0.0])) and torch.allclose(mixed[1, 0], torch.tensor([0.75, -0.75]))
    b = plain_distance_bias(4, torch.tensor([2.0]), torch.tensor([0.5]))
    assert b[0, 3, 3] == 0 and torch.allclose(b[0, 3, 1], torch.tensor(2.0 * math.log(2.0)))


def test_rotation_and_convolution_by_hand():
    x = torch.zeros(3, 1, 6)
    x[:, 0, 0], x[:, 0, 5] = 1.0, 7.0  # dimension 0 pairs with dimension 2 of four; 4 and 5 pass
    y = plain_rotate(x, 100.0, 4)
    for p in range(3):
        assert torch.allclose(y[p, 0], torch.tensor([math.cos(p), 0.0, math.sin(p), 0.0, 0.0, 7.0]), atol=1e-6)
    u = torch.tensor([[1.0], [10.0], [100.0]])
    y = plain_conv(u, torch.tensor([[3.0, 2.0, 1.0]]), torch.tensor([0.5]))
    assert y.flatten().tolist() == [1.5, 12.5, 123.5]


def test_recurrences_by_hand():
    # a decay of one half a token: log a = -8 r softplus(lam)
    lam = torch.log(torch.expm1(torch.tensor([math.log(2.0) / 8])))
    u, one = torch.tensor([[1.0], [0.0], [2.0]]), torch.ones(3, 1)
    S = plain_lru(u, one, one, lam)
    c = math.sqrt(0.75)
    assert torch.allclose(S.flatten(), torch.tensor([c, c / 2, c / 4 + 2 * c]), atol=1e-6)
    # the delta rule: a second write on the same key replaces what the first left, in proportion to beta
    k = torch.tensor([[1.0, 0.0], [1.0, 0.0], [0.0, 1.0]])
    v = torch.tensor([[2.0], [6.0], [5.0]])
    o = plain_delta_rule(torch.ones(3, 2), k, v, torch.tensor([1.0, 1.0, 0.5]), torch.tensor([1.0, 0.5, 1.0]))
    assert o.flatten().tolist() == [2.0, 4.0, 2.0 + 5.0]
    assert torch.allclose(plain_unit(torch.tensor([3.0, 4.0])), torch.tensor([0.6, 0.8]), atol=1e-6)
    assert torch.allclose(plain_gelu(torch.tensor([1.0])), torch.nn.functional.gelu(torch.tensor([1.0]), approximate="tanh"))


def test_feed_forward_by_hand():
    w = {"e.gate": torch.tensor([[3.0], [-1.0]]), "e.up": torch.tensor([[-9.0], [0.5]]), "e.down": torch.eye(2)}
    y = plain_feed_forward(torch.ones(1, 1), w, "e", 2.0, torch.float32)
    want = torch.tensor([[2.0 / (1 + math.exp(-1.702 * 2.0)) * (-2.0 + 1), -1.0 / (1 + math.exp(1.702)) * 1.5]])
    assert torch.allclose(y, want, atol=1e-6)


def test_every_mechanism_moves_the_logits():
    """The random weights of these tests are large enough that leaving a mechanism out shows."""
    toks = torch.randint(0, TRIO["vocab"], (60,), generator=torch.Generator().manual_seed(4)).tolist()
    w = plain_weights(TRIO, 1)
    base = plain_forward(w, TRIO, toks)
    scale = float(base.abs().max())

    def moved(change_w=None, change_c=None):
        w2, c2 = {k: v.clone() for k, v in w.items()}, copy.deepcopy(TRIO)
        if change_w:
            change_w(w2)
        if change_c:
            change_c(c2)
        return float((plain_forward(w2, c2, toks) - base).abs().max()) / scale

    for name in ("l0.mix.left.talk", "l0.mix.left.q.norm", "l0.mix.left.k.norm", "l0.mix.right.ra", "l0.mix.right.ri",
                 "l0.mix.right.lam", "l0.mix.right.conv.b", "l0.mix.right.x.b", "l0.mix.right.y.b", "l1.mix.A_log",
                 "l1.mix.dt_bias", "l1.mix.b", "l1.mix.norm", "l2.mix.r1", "l2.mix.r2", "l2.mix.g", "l0.ls1", "l2.ls2", "l1.norm1"):
        assert moved(lambda w2: w2[name].add_(0.5)) > 1e-3, name
    for name in ("l0.mix.right.conv", "l1.mix.q.conv", "l1.mix.k.conv", "l1.mix.v.conv", "l2.mix.q.conv", "l2.mix.k.conv"):
        assert moved(lambda w2: w2[name][:, 0].zero_()) > 1e-3, name
    left = lambda c: c["layers"][0]["mixer"]["left"]
    assert moved(change_c=lambda c: left(c)["mask"].update(size=19)) > 1e-3
    assert moved(change_c=lambda c: left(c).update(softcap=2.0)) > 1e-3
    assert moved(change_c=lambda c: left(c)["rot"].update(base=50.0)) > 1e-3
    assert moved(change_c=lambda c: c["layers"][2]["mixer"]["mask"].update(size=24)) > 1e-4
    assert moved(change_c=lambda c: c["layers"][0]["mixer"].update(right_scale=0.5)) > 1e-3
    assert moved(change_c=lambda c: c.update(residual_mult=0.6)) > 1e-3
    assert moved(change_c=lambda c: c["embedding"].update(scale=2.0)) > 1e-3
    assert moved(change_c=lambda c: c["layers"][1]["mlp"].update(limit=0.5)) > 1e-3


# ------------------------------------------------- the kernels' twins against the plain mechanisms
def _conv(C, K, T, lens, slots, seed, pad=0):
    """Convolution operands for sequences of ``lens`` tokens; the slots hold earlier inputs."""
    g = torch.Generator().manual_seed(seed)
    q_start = torch.tensor([0] + torch.tensor(lens).cumsum(0).tolist(), dtype=torch.int32)
    state = torch.randn(6, C, K - 1 + pad, generator=g)
    return ops.ConvInputs(torch.randn(C, K, generator=g), state, pad, torch.tensor(slots, dtype=torch.int32),
                          torch.repeat_interleave(torch.arange(len(lens)), torch.tensor(lens)).to(torch.int32), q_start, False)


def test_twin_of_the_scaled_addition():
    g = torch.Generator().manual_seed(0)
    h, d, s, w = torch.randn(4, 10, generator=g), torch.randn(4, 10, generator=g), torch.randn(10, generator=g), torch.rand(10, generator=g)
    for delta in (d, torch.stack([d - 1.0, torch.ones_like(d)])):
        hh, out = h.clone(), torch.empty(4, 10)
        twins.add_rmsnorm(hh, delta, w, 1e-5, out, None, s)
        torch.testing.assert_close(hh, h + d * s)
        torch.testing.assert_close(out, plain_rms(h + d * s, w, 1e-5))
        hh = h.clone()
        torch.testing.assert_close(twins.stream_add(hh, delta, None, None, s), h + d * s)


def test_twins_of_the_convolved_rows():
    """A sequence in two steps through the state's tail is the sequence in one."""
    C, K, n = 6, 4, 11
    x = torch.randn(n, C + 3, generator=torch.Generator().manual_seed(1))
    conv = _conv(C, K, n, [n], [2], 2)
    conv.state.zero_()
    want = plain_conv(x[:, :C], conv.taps)
    got = []
    for a, b in ((0, 2), (2, 3), (3, 11)):
        c = ops.ConvInputs(conv.taps, conv.state, 0, conv.slot_ids, torch.zeros(b - a, dtype=torch.int32),
                           torch.tensor([0, b - a], dtype=torch.int32), False)
        got.append(twins._convolved(x[a:b], c))
        twins.conv_tail(x[a:b], c, 1)
    torch.testing.assert_close(torch.cat(got), want)
    torch.testing.assert_close(conv.state[2].T, x[-(K - 1) :, :C])
    # an input bias is in the tail, and is no input before the start
    bias = torch.randn(C, generator=torch.Generator().manual_seed(3))
    state, out = torch.zeros(3, C, K), torch.empty(n, C)
    twins.causal_conv(x, conv.taps, None, state, 1, torch.tensor([1], dtype=torch.int32), torch.zeros(n, dtype=torch.int32),
                      torch.tensor([0, n], dtype=torch.int32), out, None, bias)
    torch.testing.assert_close(out, plain_conv(x[:, :C] + bias, conv.taps))


def test_twin_of_the_prepared_heads_with_norms_over_whole_projections():
    T, H, G, d, P = 5, 3, 1, 6, 8
    g = torch.Generator().manual_seed(5)
    src = torch.randn(T, (H + G) * d + G * 4, generator=g)
    qn, kn = torch.rand(H * d, generator=g), torch.rand(G * d, generator=g)
    q, kp, vp = torch.zeros(T, H * d), torch.zeros(2, G, P, 8), torch.zeros(2, G, 8, P)
    twins.heads_prepare(src, None, 1e-5, n_q=H, q_col=0, q_width=d, q_norm=qn, q_norm_dims=d, q_out=q, q_out_width=d, n_kv=G,
                        k_col=H * d, k_width=d, k_norm=kn, k_norm_dims=d, v_col=(H + G) * d, v_width=4,
                        slots=torch.arange(T, dtype=torch.int32), k_pages=kp, v_pages=vp, row_norm=True)
    torch.testing.assert_close(q, plain_rms(src[:, : H * d], qn, 1e-5))
    want = torch.zeros(P, G, 8)
    want[:T, 0, :d] = plain_rms(src[:, H * d : (H + G) * d], kn, 1e-5)
    torch.testing.assert_close(kp[0], pack_k(want.permute(1, 0, 2)[None])[0])


def _paged(k, v, P):
    n, G, hd = k.shape
    n_pages = -(-n // P)
    pad = torch.zeros(n_pages * P - n, G, hd)
    to = lambda x: torch.cat([x, pad]).view(n_pages, P, G, hd).permute(0, 2, 1, 3).contiguous()
    return pack_k(to(k)), pack_v(to(v)), torch.arange(n_pages, dtype=torch.int32)[None]


@pytest.mark.parametrize("window,cap", [(0, 0.0), (7, 3.0), (16, 0.0)])
def test_twin_of_attention_with_mixed_heads(window, cap):
    n, H, G, d, e, P = 40, 6, 2, 8, 8, 16
    g = torch.Generator().manual_seed(window)
    q, k, v = torch.randn(n, H, d, generator=g), torch.randn(n, G, d, generator=g), torch.randn(n, G, e, generator=g)
    talk = torch.randn(H, H, generator=g)
    kp, vp, bt = _paged(k, v, P)
    out = torch.empty(n, H * e)
    twins.mixed_attention(q.view(n, -1), d, out, e, kp, vp, bt, torch.zeros(n, dtype=torch.int32), torch.arange(n, dtype=torch.int32),
                          H, 0.4, talk, cap, window, 0.5)
    a = plain_weights_of(plain_softcap(plain_scores(q, k, 0.4), cap), plain_window(n, window))
    torch.testing.assert_close(out, 0.5 * plain_heads_attend(plain_mix_heads(a, talk), v, torch.float32), rtol=1e-4, atol=1e-5)
    single, runs = ops.mixed_attention_items([1, 0 + 19], [0, 1], [30, 21])
    assert single.tolist() == [[0, 0, 1, 30]] and sorted(r[1:3] for r in runs.tolist()) == [[1, 16], [17, 3]]
    got = torch.full((20, H * e), float("nan"))
    rows = torch.cat([q[30:31], q[21:]]).view(20, -1)
    twins.mixed_attention_mfma(rows, d, got, e, kp, vp, bt.expand(2, -1), torch.tensor(single), torch.tensor(runs), n, H, 0.4, talk,
                               cap, window, 0.5)
    torch.testing.assert_close(got, torch.cat([out[30:31], out[21:]]))


def test_twin_of_attention_with_a_distance_bias():
    n, H, G, d, P = 30, 4, 1, 8, 8
    g = torch.Generator().manual_seed(8)
    q, k = torch.randn(n, H, d, generator=g), torch.randn(n, G, d, generator=g)
    dist = torch.rand(H, 2, generator=g)
    kp, vp, bt = _paged(k, k, P)
    out = torch.empty(n, H * d)
    twins.paged_attention_general(q.view(n, -1), out, kp, vp, bt, torch.zeros(n, dtype=torch.int32), torch.arange(n, dtype=torch.int32),
                                  H, 0.3, 9, torch.zeros(H), dist)
    s = plain_scores(q, k, 0.3) - plain_distance_bias(n, dist[:, 0], dist[:, 1])
    torch.testing.assert_close(out, plain_heads_attend(plain_weights_of(s, plain_window(n, 9), True), k, torch.float32), rtol=1e-4, atol=1e-5)


def test_twins_of_the_delta_rule():
    G, d, H, e, K = 2, 6, 4, 8, 3
    C, lens = 2 * G * d + H * e, [7, 1, 4]
    T = sum(lens)
    g = torch.Generator().manual_seed(9)
    src = torch.randn(T, C + 2 * H + 1, generator=g)
    rate, dt = torch.rand(H, generator=g), torch.randn(H, generator=g)
    conv = _conv(C, K, T, lens, [4, 0, 3], 10)
    conv.state.zero_()
    ready = torch.empty(T, C + 2 * H)
    twins.delta_prepare(src, G, d, H, e, conv, C, C + H, rate, dt, d ** -0.5, 1e-6, ready)
    state, out = torch.zeros(6, H, d, e), torch.empty(T, H * e)
    twins.delta_scan(ready, G, d, H, e, state, conv.slot_ids, conv.q_start, 3, out)
    for b, n in enumerate(lens):
        r = src[int(conv.q_start[b]) :][:n]
        y = plain_silu(plain_conv(r[:, :C], conv.taps))
        q = plain_unit(y[:, : G * d].view(n, G, d)) * d ** -0.5
        k = plain_unit(y[:, G * d : 2 * G * d].view(n, G, d))
        v = y[:, 2 * G * d :].view(n, H, e)
        decay = torch.exp(-rate * torch.nn.functional.softplus(r[:, C + H : C + 2 * H] + dt))
        beta = torch.sigmoid(r[:, C : C + H])
        want = torch.stack([plain_delta_rule(q[:, h // 2], k[:, h // 2], v[:, h], decay[:, h], beta[:, h]) for h in range(H)], 1)
        torch.testing.assert_close(out[int(conv.q_start[b]) :][:n], want.reshape(n, -1), rtol=1e-5, atol=1e-5)


def test_twin_of_the_linear_recurrence():
    B, n, K, lens = 3, 4, 3, [6, 1]
    C, T = B * n, 7
    g = torch.Generator().manual_seed(11)
    u, y, x = torch.randn(T, C, generator=g), torch.randn(T, C, generator=g), torch.randn(T, C, generator=g)
    w, bias = torch.randn(B, 2 * n, n, generator=g), torch.randn(B, 2 * n, generator=g)
    gates = torch.empty(T, 2 * C)
    twins.head_linear(u, n, w, gates, 2 * n, bias=bias)
    lam, yb, xb = torch.randn(C, generator=g), torch.randn(C, generator=g), torch.randn(C, generator=g)
    decay = 8.0 * torch.nn.functional.softplus(lam)
    state, out = torch.zeros(4, C, K), torch.empty(T, C)
    twins.lru_scan(u, gates, n, decay, y, yb, 0.5, x, xb, K, state, torch.tensor([3, 1], dtype=torch.int32),
                   torch.tensor([0, 6, 7], dtype=torch.int32), 2, out)
    r = torch.sigmoid(plain_block_linear(u, w[:, :n], bias[:, :n], torch.float32))
    i = torch.sigmoid(plain_block_linear(u, w[:, n:], bias[:, n:], torch.float32))
    for a, b, slot in ((0, 6, 3), (6, 7, 1)):
        S = plain_lru(u[a:b], r[a:b], i[a:b], lam)
        torch.testing.assert_close(out[a:b], 0.5 * S * plain_gelu(y[a:b] + yb), rtol=1e-5, atol=1e-5)
        torch.testing.assert_close(state[slot, :, 0], S[-1], rtol=1e-5, atol=1e-5)
    torch.testing.assert_close(state[3, :, 1:].T, x[4:6] + xb)
    torch.testing.assert_close(state[1, :, 1:].T, torch.stack([torch.zeros(C), x[6] + xb]))


def test_a_whole_model_in_float64_and_float32_agree():
    for config in (TRIO, ODD, WIDE):
        w = plain_weights(config, 3)
        toks = [t % config["vocab"] for t in range(5, 45)]
        a, b = plain_forward(w, config, toks, torch.float64), plain_forward(w, config, toks)
        assert float((a - b.double()).abs().max()) < 1e-4 * float(a.abs().max())
