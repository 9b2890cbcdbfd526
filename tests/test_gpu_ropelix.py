"""Ropelix on the GPU against the plain implementation (``tests/plain_ropelix.py``) and the kernels' plain twins: each
new kernel alone, then whole models of several shapes under every way of cutting requests into steps, with small pools
so that pages and slots change hands, in float32 (strict) and bfloat16."""

from __future__ import annotations

import copy
from typing import Dict, List

import pytest
import torch

import traces
from helpers import assert_close, make_runner, run_trace, save_model_folder
from plain_ropelix import (ODD, ONLY_CONV, ONLY_DELTA, ONLY_MIXED, TRIO, WIDE, plain_forward, plain_greedy, plain_weights)

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
CONFIGS = {"trio": TRIO, "odd": ODD, "wide": WIDE, "only_mixed": ONLY_MIXED, "only_conv": ONLY_CONV, "only_delta": ONLY_DELTA}


def _tokens(config, lengths: Dict[str, int], seed: int) -> Dict[str, List[int]]:
    g = torch.Generator().manual_seed(seed)
    return {r: torch.randint(0, config["vocab"], (n,), generator=g).tolist() for r, n in lengths.items()}


def _close(got, want, dtype, what="", scale=1.0):
    tol = dict(rtol=2e-5, atol=2e-5 * scale) if dtype == torch.float32 else dict(rtol=2e-2, atol=2e-2 * scale)
    torch.testing.assert_close(got.float().cpu(), want.float().cpu(), msg=lambda m: f"{what}: {m}", **tol)


def _dev(x):
    return x.to(DEV).contiguous()


# ------------------------------------------------------------------ kernels alone
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,D", [(5, 42), (7, 200), (3, 2304), (4, 4096), (2, 8200)])
def test_scaled_addition_and_norm(dtype, T, D):
    from fastgen_amd.kernels import ops, twins

    g = torch.Generator().manual_seed(T + D)
    h, w, s = torch.randn(T, D, generator=g), torch.rand(D, generator=g) + 0.5, torch.randn(D, generator=g)
    rows = torch.tensor([T - 1, 0, T - 1], dtype=torch.int32)
    for delta in (torch.randn(T, D, generator=g).to(dtype), torch.randn(3, T, D, generator=g), torch.randn(9, T, D, generator=g)):
        hc, hg = h.clone(), _dev(h)
        oc, og = torch.empty(T, D, dtype=dtype), torch.empty(T, D, dtype=dtype, device=DEV)
        gc, gg = torch.empty(3, D, dtype=dtype), torch.empty(3, D, dtype=dtype, device=DEV)
        twins.add_rmsnorm(hc.clone(), delta, w, 1e-5, gc, rows, s)
        ops.add_rmsnorm(hg, _dev(delta), _dev(w), 1e-5, gg, _dev(rows), _dev(s))
        assert torch.equal(hg.cpu(), h)
        twins.add_rmsnorm(hc, delta, w, 1e-5, oc, None, s)
        ops.add_rmsnorm(hg, _dev(delta), _dev(w), 1e-5, og, None, _dev(s))
        _close(hg, hc, torch.float32, "stream", 4.0)
        _close(og, oc, dtype, "normed")
        _close(gg, gc, dtype, "gathered")
        hg = _dev(h)
        ops.stream_add(hg, _dev(delta), None, None, _dev(s))
        _close(hg, hc, torch.float32, "stream_add", 4.0)


def _conv_inputs(C, K, lens, moves, seed, device="cpu", pad=0, slots=8):
    from fastgen_amd.kernels import ops

    g = torch.Generator().manual_seed(seed)
    B = len(lens)
    q_start = torch.tensor([0] + torch.tensor(lens).cumsum(0).tolist(), dtype=torch.int32)
    seq = torch.repeat_interleave(torch.arange(B), torch.tensor(lens)).to(torch.int32)
    slot_ids = torch.randperm(slots, generator=g)[:B].to(torch.int32)
    state = torch.randn(slots, C, max(1, K - 1) + pad, generator=g)
    taps = torch.randn(C, K, generator=g)
    to = lambda x: x.to(device).contiguous()
    return ops.ConvInputs(to(taps), to(state), pad, to(slot_ids), to(seq), to(q_start), moves)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("lens", [(9, 1, 4), (1, 1, 1)])
@pytest.mark.parametrize("H,G,d,hc,K,P", [(4, 2, 16, 16, 4, 16), (3, 1, 20, 32, 1, 8), (2, 2, 96, 96, 2, 64)])
def test_heads_behind_a_convolution(dtype, lens, H, G, d, hc, K, P):
    from fastgen_amd.kernels import ops, twins

    T, C = sum(lens), (H + G) * d
    src = torch.randn(T, C + 5, generator=torch.Generator().manual_seed(K))
    slots = torch.randperm(3 * P, generator=torch.Generator().manual_seed(1))[:T].to(torch.int32)
    moves = max(lens) == 1
    res = []
    for dev, fn in (("cpu", twins), (DEV, ops)):
        conv = _conv_inputs(C, K, lens, moves, 3, dev)
        kp, vp = torch.zeros(3, G, P, hc, dtype=dtype, device=dev), torch.zeros(3, G, hc, P, dtype=dtype, device=dev)
        q = torch.zeros(T, H * hc, dtype=dtype, device=dev)
        x = src.to(dev)
        fn.heads_prepare(x, None, 0.0, n_q=H, q_col=0, q_width=d, q_out=q, q_out_width=hc, n_kv=G, k_col=H * d, k_width=d,
                         v_col=-1, v_width=d, slots=slots.to(dev), k_pages=kp, v_pages=vp, conv=conv)
        if not moves:
            fn.conv_tail(x, conv, len(lens))
        res.append((q, kp, vp, conv.state))
    for a, b, what in zip(res[1], res[0], ("queries", "keys", "values", "tails")):
        _close(a, b, torch.float32 if what == "tails" else dtype, what)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,d,e,rot,P", [(4, 2, 16, 24, 8, 16), (20, 4, 8, 8, 4, 8), (3, 3, 12, 6, 0, 64)])
def test_heads_with_norms_over_whole_projections(dtype, H, G, d, e, rot, P):
    from fastgen_amd.kernels import ops, twins

    T, hc = 11, -(-max(d, e) // 16) * 16
    g = torch.Generator().manual_seed(H)
    src = torch.randn(T, (H + G) * d + G * e, generator=g)
    qn, kn = torch.rand(H * d, generator=g) + 0.5, torch.rand(G * d, generator=g) + 0.5
    slots = torch.randperm(3 * P, generator=g)[:T].to(torch.int32)
    slots[4] = -1
    table = torch.randn(T, rot // 2, 2, generator=g) if rot else None
    res = []
    for dev, fn in (("cpu", twins), (DEV, ops)):
        kp, vp = torch.zeros(3, G, P, hc, dtype=dtype, device=dev), torch.zeros(3, G, hc, P, dtype=dtype, device=dev)
        q = torch.zeros(T, H * d, dtype=dtype, device=dev)
        to = lambda x: x.to(dev) if x is not None else None
        fn.heads_prepare(to(src), None, 1e-5, n_q=H, q_col=0, q_width=d, q_norm=to(qn), q_norm_dims=d, q_out=q, q_out_width=d,
                         n_kv=G, k_col=H * d, k_width=d, k_norm=to(kn), k_norm_dims=d, v_col=(H + G) * d, v_width=e,
                         table=to(table), rotary_dim=rot, slots=to(slots), k_pages=kp, v_pages=vp, row_norm=True)
        res.append((q, kp, vp))
    for a, b, what in zip(res[1], res[0], ("queries", "keys", "values")):
        _close(a, b, dtype, what)


def _random_pages(n, G, d, e, P, dtype, seed):
    """Keys and values of one sequence of ``n`` tokens in shuffled pages; everything else in the pools is NaN."""
    from fastgen_amd.cache.layout import pack_k, pack_v

    g = torch.Generator().manual_seed(seed)
    hd, n_pages = -(-max(d, e) // 16) * 16, -(-n // P)
    k, v = torch.zeros(n_pages * P, G, hd), torch.zeros(n_pages * P, G, hd)
    k[:n, :, :d], v[:n, :, :e] = torch.randn(n, G, d, generator=g), torch.randn(n, G, e, generator=g)
    k[n:], v[n:] = float("nan"), float("nan")
    to = lambda x: x.to(dtype).view(n_pages, P, G, hd).permute(0, 2, 1, 3).contiguous()
    where = torch.randperm(n_pages + 2, generator=g)[:n_pages]
    kp = torch.full((n_pages + 2, G, P, hd), float("nan"), dtype=dtype)
    vp = torch.full((n_pages + 2, G, hd, P), float("nan"), dtype=dtype)
    kp[where], vp[where] = pack_k(to(k)), pack_v(to(v))
    return k[:n, :, :d].to(dtype), v[:n, :, :e].to(dtype), kp, vp, where.int()[None]


MIXED = [(4, 2, 16, 24, 150, 64, 20, 8.0), (6, 3, 96, 64, 230, 64, 0, 0.0), (16, 4, 128, 128, 333, 64, 100, 30.0),
         (12, 12, 32, 16, 130, 32, 33, 0.0), (15, 5, 24, 40, 200, 32, 64, 5.0), (16, 1, 32, 32, 700, 64, 0, 10.0),
         (1, 1, 16, 16, 70, 32, 1, 0.0), (10, 2, 160, 176, 140, 64, 50, 4.0), (16, 16, 256, 208, 90, 64, 40, 8.0), (20, 4, 8, 8, 90, 16, 16, 3.0), (3, 3, 12, 6, 75, 8, 0, 0.0)]


@pytest.mark.parametrize("H,G,d,e,n,P,window,cap", MIXED)
def test_attention_with_mixed_heads(H, G, d, e, n, P, window, cap):
    """The general kernel in both precisions and the matrix-core kernels (a prompt, and every token decoded alone)
    against the formula; free pages and slots hold NaN."""
    from fastgen_amd.kernels import ops

    g = torch.Generator().manual_seed(n)
    i = torch.arange(n)
    vis = (i[:, None] >= i[None]) & ((i[:, None] - i[None] < window) if window else True)
    for dtype in (torch.float32, torch.bfloat16):
        k, v, kp, vp, bt = _random_pages(n, G, d, e, P, dtype, n)
        q = (2 * torch.randn(n, H * d, generator=g)).to(dtype)
        talk = torch.eye(H) + 0.3 * torch.randn(H, H, generator=g)
        s = torch.einsum("thd,jhd->htj", q.float().view(n, H, d), k.float().repeat_interleave(H // G, 1)) * d ** -0.5
        s = cap * torch.tanh(s / cap) if cap else s
        a = torch.einsum("hg,gtj->htj", talk, torch.softmax(s.masked_fill(~vis, float("-inf")), -1))
        want = 0.7 * torch.einsum("htj,jhe->the", a, v.float().repeat_interleave(H // G, 1)).reshape(n, -1)
        out = torch.full((n, H * e), float("nan"), dtype=dtype, device=DEV)
        args = (_dev(kp), _dev(vp), _dev(bt))
        ops.mixed_attention(_dev(q), d, out, e, *args, torch.zeros(n, dtype=torch.int32, device=DEV), _dev(i.int()), H, d ** -0.5,
                            _dev(talk), cap, window, 0.7)
        _close(out, want, dtype, "general kernel")
        if dtype == torch.float32 or not ops.mixed_attention_mfma_ok(dtype, H, kp.shape[3], P):
            continue
        for exact in (False, True):  # a matrix that bfloat16 holds, and one that it does not
            t = talk if not exact else talk.to(torch.bfloat16).float()
            ref = want if not exact else 0.7 * torch.einsum(
                "htj,jhe->the", torch.einsum("hg,gtj->htj", t, torch.softmax(s.masked_fill(~vis, float("-inf")), -1)),
                v.float().repeat_interleave(H // G, 1)).reshape(n, -1)
            _, runs = ops.mixed_attention_items([n], [0], [0])
            out.fill_(float("nan"))
            ops.mixed_attention_mfma(_dev(q), d, out, e, *args, None, _dev(torch.tensor(runs)), n, H, d ** -0.5, _dev(t), cap, window,
                                     0.7, not exact)
            _close(out, ref, dtype, "prompt on the matrix cores")
            single = torch.stack([torch.zeros(n), i, torch.ones(n), i], 1).int()
            out.fill_(float("nan"))
            ops.mixed_attention_mfma(_dev(q), d, out, e, *args, _dev(single), None, n, H, d ** -0.5, _dev(t), cap, window, 0.7, not exact)
            _close(out, ref, dtype, "decoded on the matrix cores")
        # portions and single tokens in one call, as two sequences over the same pages
        cut = n - 37
        single, runs = ops.mixed_attention_items([1, 37], [0, 1], [n - 1, cut])
        rows = torch.cat([q[n - 1 :], q[cut:]])
        both = torch.full((38, H * e), float("nan"), dtype=dtype, device=DEV)
        ops.mixed_attention_mfma(_dev(rows), d, both, e, *args[:2], _dev(bt.expand(2, -1)), _dev(torch.tensor(single)),
                                 _dev(torch.tensor(runs)), n, H, d ** -0.5, _dev(talk), cap, window, 0.7)
        _close(both, torch.cat([want[n - 1 :], want[cut:]]), dtype, "portion beside a single token")


@pytest.mark.parametrize("H,G,d,n,P,window", [(4, 1, 16, 150, 64, 32), (8, 2, 96, 300, 64, 70), (20, 1, 16, 90, 16, 16), (3, 3, 32, 130, 32, 0)])
def test_attention_with_a_distance_bias(H, G, d, n, P, window):
    from fastgen_amd.kernels import ops

    g = torch.Generator().manual_seed(d)
    i = torch.arange(n)
    far = (i[:, None] - i[None]).clamp(min=0).float()
    vis = (i[:, None] >= i[None]) & ((i[:, None] - i[None] < window) if window else True)
    dist = torch.stack([0.2 + torch.rand(H, generator=g), 0.05 + torch.rand(H, generator=g)], 1)
    for dtype in (torch.float32, torch.bfloat16):
        k, v, kp, vp, bt = _random_pages(n, G, d, d, P, dtype, n)
        q = (2 * torch.randn(n, H * d, generator=g)).to(dtype)
        s = torch.einsum("thd,jhd->htj", q.float().view(n, H, d), k.float().repeat_interleave(H // G, 1)) * d ** -0.5
        s = s - dist[:, 0, None, None] * torch.log1p(dist[:, 1, None, None] * far)
        e = torch.where(vis, torch.exp(s), torch.zeros(()))
        want = torch.einsum("htj,jhd->thd", e / (1 + e.sum(-1, keepdim=True)), v.float().repeat_interleave(H // G, 1)).reshape(n, -1)
        args, sinks = (_dev(kp), _dev(vp), _dev(bt)), torch.zeros(H, device=DEV)
        out = torch.full((n, H * d), float("nan"), dtype=dtype, device=DEV)
        ops.paged_attention_general(_dev(q), out, *args, torch.zeros(n, dtype=torch.int32, device=DEV), _dev(i.int()), H, d ** -0.5,
                                    window, sinks, _dev(dist))
        _close(out, want, dtype, "general kernel")
        if dtype == torch.float32 or H // G > 16:
            continue
        per = max(1, ops.attention_tile_rows(d, False, True, True) // (H // G))
        big = torch.tensor([[0, a, min(per, n - a), a] for a in range(0, n, per)], dtype=torch.int32)
        out.fill_(float("nan"))
        ops.paged_attention_mfma(_dev(q), out, *args, None, _dev(big), H, d ** -0.5, window, exact_weights=True, sinks=sinks,
                                 distance=_dev(dist))
        _close(out, want, dtype, "tiles")
        small = torch.stack([torch.zeros(n), i, torch.ones(n), i], 1).int()
        out.fill_(float("nan"))
        ops.paged_attention_mfma(_dev(q), out, *args, _dev(small), None, H, d ** -0.5, window, exact_weights=True, sinks=sinks,
                                 distance=_dev(dist))
        _close(out, want, dtype, "split keys")


@pytest.mark.parametrize("lens", [(200, 1, 70), (64, 65), (63, 5, 1), (1, 1, 1, 1), (131,)])
@pytest.mark.parametrize("G,d,H,e,K", [(2, 16, 4, 24, 3), (1, 64, 3, 32, 4), (3, 10, 6, 14, 2), (2, 128, 2, 128, 2), (1, 48, 1, 16, 1),
                                       (1, 272, 2, 20, 2), (2, 176, 4, 40, 2)])
def test_delta_rule_token_by_token_and_in_chunks(lens, G, d, H, e, K):
    """Preparation and scan against the twins run in float64; the scan alone, and (with the lengths on the host) in
    chunks.  Decays reach from a forgotten state to one that never fades."""
    from fastgen_amd.kernels import ops, twins

    C, T, B = 2 * G * d + H * e, sum(lens), len(lens)
    g = torch.Generator().manual_seed(d + T)
    src = torch.randn(T, C + 2 * H + 3, generator=g)
    src[:, C + H : C + 2 * H] = 6 * torch.randn(T, H, generator=g)
    rate, dt = torch.rand(H, generator=g), torch.randn(H, generator=g)
    moves = max(lens) == 1
    width = -(-(C + 2 * H) // 4) * 4
    cc, cg = _conv_inputs(C, K, lens, moves, 7), _conv_inputs(C, K, lens, moves, 7, DEV)
    rc, rg = torch.zeros(T, width), torch.zeros(T, width, device=DEV)
    twins.delta_prepare(src, G, d, H, e, cc, C, C + H, rate, dt, d ** -0.5, 1e-6, rc)
    ops.delta_prepare(_dev(src), G, d, H, e, cg, C, C + H, _dev(rate), _dev(dt), d ** -0.5, 1e-6, rg)
    _close(rg, rc, torch.float32, "prepared rows", 4.0)
    if not moves:
        twins.conv_tail(src, cc, B)
        ops.conv_tail(_dev(src), cg, B)
    _close(cg.state, cc.state, torch.float32, "tails")
    state = torch.randn(8, H * d * e + 6, generator=g)  # (slots with a stride of their own)
    view = lambda s: s[:, : H * d * e].view(8, H, d, e)
    sc, oc = state.double(), torch.empty(T, H * e, dtype=torch.float64)
    twins.delta_scan(rc.double(), G, d, H, e, view(sc), cc.slot_ids, cc.q_start, B, oc)
    for host in (None, cc.q_start.numpy()):
        sg, og = _dev(state), torch.full((T, H * e), float("nan"), device=DEV)
        ops.delta_scan(_dev(rc), G, d, H, e, view(sg), cg.slot_ids, cg.q_start, B, og, host)
        what = "token by token" if host is None else "chunks"
        scale = max(1.0, float(oc.abs().max()))
        assert float((og.double().cpu() - oc).abs().max()) <= 2e-5 * scale, what
        assert float((sg.double().cpu() - sc).abs().max()) <= 2e-5 * max(1.0, float(sc.abs().max())), f"{what}: state"


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("lens", [(200, 1, 70), (95, 3), (1, 1, 1)])
@pytest.mark.parametrize("blocks,n,K", [(3, 16, 4), (1, 36, 1), (4, 20, 2), (2, 136, 5)])
def test_linear_recurrence_token_by_token_and_in_chunks(dtype, lens, blocks, n, K):
    from fastgen_amd.kernels import ops, twins

    C, T, B = blocks * n, sum(lens), len(lens)
    g = torch.Generator().manual_seed(C + T)
    x, y = torch.randn(T, C + 4, generator=g), torch.randn(T, C + 4, generator=g)
    xb, yb, cb = torch.randn(C, generator=g), torch.randn(C, generator=g), torch.randn(C, generator=g)
    conv = _conv_inputs(C, K, lens, False, 5, pad=1)
    state = torch.randn(8, C, K, generator=g)
    u_c, u_g = torch.empty(T, C, dtype=dtype), torch.empty(T, -(-C // 8) * 8, dtype=dtype, device=DEV)
    twins.causal_conv(x, conv.taps, cb, state, 1, conv.slot_ids, conv.seq_of_token, conv.q_start, u_c, None, xb)
    ops.causal_conv(_dev(x), _dev(conv.taps), _dev(cb), _dev(state), 1, _dev(conv.slot_ids), _dev(conv.seq_of_token), _dev(conv.q_start),
                    u_g, None, _dev(xb))
    _close(u_g[:, :C], u_c, dtype, "convolution", 4.0)
    u_g[:, :C] = _dev(u_c)  # (what follows from equal inputs)
    w, gb = (torch.randn(blocks, 2 * n, n, generator=g) * n ** -0.5).to(dtype), torch.randn(blocks, 2 * n, generator=g)
    gates_c, gates_g = torch.empty(T, 2 * C), torch.empty(T, 2 * C, device=DEV)
    twins.head_linear(u_c, n, w, gates_c, 2 * n, bias=gb)
    ops.head_linear(u_g, n, _dev(w), gates_g, 2 * n, bias=_dev(gb))
    _close(gates_g, gates_c, torch.float32, "gates", 4.0)
    decay = 8.0 * torch.nn.functional.softplus(torch.randn(C, generator=g) * 3 - 4)
    s_c, o_c = state.clone(), torch.empty(T, C, dtype=dtype)
    twins.lru_scan(u_c, gates_c, n, decay, y, yb, 0.6, x, xb, K, s_c, conv.slot_ids, conv.q_start, B, o_c)
    for host in (None, conv.q_start.numpy()):
        s_g, o_g = _dev(state), torch.empty(T, C + 3, dtype=dtype, device=DEV)
        ops.lru_scan(u_g, _dev(gates_c), n, _dev(decay), _dev(y), _dev(yb), 0.6, _dev(x), _dev(xb), K, s_g, _dev(conv.slot_ids),
                     _dev(conv.q_start), B, o_g, host)
        what = "token by token" if host is None else "chunks"
        _close(o_g[:, :C], o_c, dtype, what, 4.0)
        _close(s_g, s_c, torch.float32 if dtype == torch.float32 else dtype, f"{what}: state", 4.0)


# ----------------------------------------------------------------- whole models
LENGTHS = {"a": 150, "b": 37, "c": 2, "d": 1, "e": 70, "f": 19}


@pytest.fixture(scope="module")
def cases(tmp_path_factory):
    out = {}
    for name, config in CONFIGS.items():
        weights = plain_weights(config, seed=len(name))
        folder = save_model_folder(tmp_path_factory.mktemp(name), config, weights)
        toks = _tokens(config, LENGTHS, seed=7)
        runs = {dt: {r: plain_forward(weights, config, t, dt) for r, t in toks.items()}
                for dt in (torch.float32, torch.float64, torch.bfloat16)}
        out[name] = (config, weights, folder, toks, runs)
    return out


def _against(got, runs, dtype, what):
    """float32: against the float64 run, three times what the plain float32 run is off at its worst.  bfloat16: the
    root mean square over all logits of all requests at most 1.3 times the plain bfloat16 run's, and no position off by
    more than four times that run's worst (single positions may stand on an edge where rounding counts for more)."""
    if dtype == torch.float32:
        want, low = runs[torch.float64], runs[torch.float32]
        level = max(float((low[r].double() - want[r]).abs().max()) for r in want)
        assert_close(got, want, dtype, {r: want[r] + level for r in want}, what)
        return
    want, low = runs[torch.float64], runs[torch.bfloat16]
    for r in want:
        assert got[r].shape == want[r].shape and torch.isfinite(got[r]).all(), f"{what} {r}"
    flat = lambda runs_: torch.cat([(runs_[r].double() - want[r]).flatten() for r in want])
    g, l = flat(got), flat(low)
    scale = max(float(want[r].abs().max()) for r in want)
    rms = lambda e: float(e.pow(2).mean().sqrt())
    assert rms(g) <= 1.3 * rms(l) + 1e-4 * scale, f"{what}: root mean square {rms(g):.3e}, the plain run's {rms(l):.3e}"
    assert float(g.abs().max()) <= 4 * float(l.abs().max()) + 1e-3 * scale, f"{what}: worst {float(g.abs().max()):.3e} against {float(l.abs().max()):.3e}"


def _all_traces(lengths):
    return {"whole": traces.whole(lengths), "tail": traces.tail(lengths, 60), "chunks": traces.chunks(lengths),
            "pairs": traces.chunks(lengths, sizes=(2, 3, 2, 5)),
            "mixed": traces.mixed(lengths, seed=3), "mixed2": traces.mixed(lengths, max_live=3, seed=11, budget=23)}


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_float32_every_cut_batch_and_reuse(cases, name):
    """Whole prompts, prompts then single tokens, portions down to two tokens and one, mixed batches of unequal
    requests: the same logits as the plain run whatever the cut.  Pages of 16 tokens and a pool that holds the live
    requests only: pages and slots are used again."""
    config, weights, folder, toks, runs = cases[name]
    runner = make_runner(folder, torch.float32, page_size=16, max_tokens=304, max_requests=4)
    first = None
    for kind, tr in _all_traces(LENGTHS).items():
        got = run_trace(runner, tr, toks)
        _against(got, runs, torch.float32, f"ropelix {name} {kind}")
        if first is None:
            first = got
        for r in got:
            assert float((got[r] - first[r]).abs().max()) <= 1e-5 * float(first[r].abs().max()), f"{name} {kind}: {r} depends on the cut"
        assert all(runner.cache.free_pages(g) == 304 // 16 for g in range(runner.cache.n_groups))
        assert runner.cache.free_slots() == 4


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_bfloat16_every_cut_batch_and_reuse(cases, name):
    config, weights, folder, toks, runs = cases[name]
    for page, pool in ((16, 304), (64, 768)):  # (pages of 64: the matrix-core kernels with mixed heads)
        runner = make_runner(folder, torch.bfloat16, page_size=page, max_tokens=pool, max_requests=4)
        for kind, tr in _all_traces(LENGTHS).items():
            _against(run_trace(runner, tr, toks), runs, torch.bfloat16, f"ropelix {name} {kind} bfloat16, pages of {page}")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_the_stream_after_every_layer(cases, dtype):
    from fastgen_amd.engine import Model, ModelRunner, StepEntry
    from fastgen_amd.kernels import ops

    config, weights, folder, toks, _ = cases["trio"]
    want: list = []
    plain_forward(weights, config, toks["b"], dtype, want)
    model = Model.from_folder(folder, dtype, DEV)
    seen = []
    for block in model.parts.blocks:
        def wrap(keep=block.forward):
            def forward(h, pending, ctx, store):
                out = keep(h, pending, ctx, store)
                after = h.clone()
                ops.stream_add(after, out.rows, None, None, out.scale)
                seen.append(after.cpu())
                return out
            return forward
        block.forward = wrap()
    runner = ModelRunner(model, page_size=16, max_tokens=64, max_requests=1)
    runner.step([StepEntry("b", toks["b"], [0])])
    assert len(seen) == len(want)
    for i, (g, w) in enumerate(zip(seen, want)):
        tol = 2e-5 if dtype == torch.float32 else 4e-2
        assert float((g - w.float()).abs().max()) <= tol * float(w.abs().max()), f"after layer {i}"


def _runs(weights, config, toks):
    return {dt: {r: plain_forward(weights, config, t, dt) for r, t in toks.items()} for dt in (torch.float32, torch.float64, torch.bfloat16)}


@pytest.mark.parametrize("name", ["trio", "odd"])
def test_long_decoding_across_pages_and_windows(cases, name):
    """A short prompt, then 290 tokens one by one over many pages and past every window (recorded steps)."""
    config, weights, folder, _, _ = cases[name]
    toks = _tokens(config, {"z": 300}, seed=5)
    runs = _runs(weights, config, toks)
    for dtype, page in ((torch.float32, 16), (torch.bfloat16, 16), (torch.bfloat16, 64)):
        runner = make_runner(folder, dtype, page_size=page, max_tokens=320, max_requests=2)
        _against(run_trace(runner, traces.tail({"z": 300}, 290), toks), runs, dtype, f"ropelix {name} long decoding {dtype}")


@pytest.mark.parametrize("name", ["trio", "wide"])
def test_long_prompts_beside_short_ones(cases, name):
    """Prompts of several hundred tokens in one step (recurrences in chunks), together in one batch, in two steps and in
    small portions."""
    config, weights, folder, _, _ = cases[name]
    lengths = {"p": 500, "q": 260, "r": 3}
    toks = _tokens(config, lengths, seed=13)
    runs = _runs(weights, config, toks)
    together = [([("p", 0, 500), ("q", 0, 260), ("r", 0, 3)], ["p", "q", "r"])]
    for dtype, page in ((torch.float32, 16), (torch.bfloat16, 16), (torch.bfloat16, 64)):
        runner = make_runner(folder, dtype, page_size=page, max_tokens=896, max_requests=3)
        for kind, tr in (("whole", traces.whole(lengths)), ("together", together),
                         ("halves", traces.chunks(lengths, sizes=(290, 210))), ("portions", traces.chunks(lengths))):
            _against(run_trace(runner, tr, toks), runs, dtype, f"ropelix {name} long {kind} {dtype}")


def test_many_sequences_decoding_together(cases):
    """Twenty requests decode side by side: recorded steps filled up with stand-in sequences, whose state is nobody's."""
    config, weights, folder, _, _ = cases["trio"]
    prompts = {f"s{i}": 3 + 5 * (i % 7) for i in range(20)}
    lengths = {r: n + 12 for r, n in prompts.items()}
    toks = _tokens(config, lengths, seed=3)
    runs = _runs(weights, config, toks)
    tr = traces.many_decoding_together(prompts, 12, seed=1)
    for dtype in (torch.float32, torch.bfloat16):
        runner = make_runner(folder, dtype, page_size=64, max_tokens=64 * 20, max_requests=20)
        _against(run_trace(runner, tr, toks), runs, dtype, f"ropelix many decoding {dtype}")


def test_keys_at_the_edges_of_windows_and_pages(tmp_path):
    """One attention layer of either kind with sharp scores and windows of 32, 16 (one page) and 21: the plain run with a
    window one token longer or shorter differs by far more than the tolerance, and the engine agrees with the right
    one, for whole prompts, portions down to two tokens and tokens decoded alone."""
    n = 130
    for base, window in ((ONLY_MIXED, 32), (ONLY_MIXED, 21), (ONLY_CONV, 16), (ONLY_CONV, 21)):
        config = copy.deepcopy(base)
        mixer = config["layers"][0]["mixer"]
        at = mixer.get("left", mixer)
        at["mask"]["size"], at["scale"] = window, 6 * at["scale"]
        w = plain_weights(config, window)
        if base is ONLY_CONV:
            w["l0.mix.r1"] *= 0.1
        toks = _tokens(config, {"s": n}, seed=window)
        runs = _runs(w, config, toks)
        want = runs[torch.float32]["s"]
        for other_size in (window - 1, window + 1):
            other = copy.deepcopy(config)
            m = other["layers"][0]["mixer"]
            m.get("left", m)["mask"]["size"] = other_size
            moved = (plain_forward(w, other, toks["s"]) - want).abs().amax(-1)
            assert float(moved[window:].max()) > 0.05 * float(want.abs().max()), "the window's edge does not decide"
        folder = save_model_folder(tmp_path / f"{config['layers'][0]['type']}{window}", config, w)
        for dtype, page in ((torch.float32, 16), (torch.bfloat16, 16), (torch.bfloat16, 64)):
            runner = make_runner(folder, dtype, page_size=page, max_tokens=192, max_requests=1)
            for kind, tr in (("whole", traces.whole({"s": n})), ("tail", traces.tail({"s": n}, 90)), ("chunks", traces.chunks({"s": n})),
                             ("pairs", traces.chunks({"s": n}, sizes=(2, 3, 2, 5)))):
                _against(run_trace(runner, tr, toks), runs, dtype, f"window {window} {kind} {dtype}")


@pytest.mark.parametrize("kind", ["delta", "lru", "sink"])
def test_a_state_that_remembers_and_a_sink_that_counts(tmp_path, kind):
    """Recurrences that hardly forget: changing the first 40 tokens of hundreds changes the last logits, whole, in portions,
    decoded alone, through slots that another request held.  The one in the softmax's denominator takes a visible share."""
    config = copy.deepcopy({"delta": ONLY_DELTA, "lru": ONLY_MIXED, "sink": ONLY_CONV}[kind])
    n = {"delta": 200, "lru": 600, "sink": 120}[kind]
    if kind == "delta":  # (keys of 64: a later write leaves most of an earlier one standing)
        config["layers"][0]["mixer"].update(dim=64)
    elif kind == "sink":
        config["layers"][0]["mixer"].update(mask={"size": 5}, scale=0.05)
        config["embedding"]["scale"] = 0.5  # (the stream is mostly what the layer added)
    w = plain_weights(config, 9)
    if kind == "delta":
        w["l0.mix.A_log"].fill_(-9.0)
    elif kind == "lru":
        w["l0.mix.right.lam"].fill_(-9.0)
        config["layers"][0]["mixer"].update(left_scale=0.1, right_scale=2.0)
    lengths = {"other": 70, "s": n}
    toks = _tokens(config, lengths, seed=2)
    runs = _runs(w, config, toks)
    want = runs[torch.float32]["s"]
    scale = float(want.abs().max())
    if kind == "sink":
        no_sink = plain_without_sink(w, config, toks["s"])
        assert float(((no_sink - want).abs().amax(-1) > 0.02 * scale).float().mean()) > 0.3, "the sink does not count"
    else:
        changed = [(t + 1) % config["vocab"] if i < 40 else t for i, t in enumerate(toks["s"])]
        assert float((plain_forward(w, config, changed)[-30:] - want[-30:]).abs().max()) > 0.02 * scale, "nothing is remembered"
    folder = save_model_folder(tmp_path / kind, config, w)
    for dtype, page in ((torch.float32, 16), (torch.bfloat16, 64)):
        runner = make_runner(folder, dtype, page_size=page, max_tokens=640, max_requests=1)
        for what, tr in (("whole", traces.whole(lengths)), ("tail", traces.tail(lengths, 40)), ("chunks", traces.chunks(lengths)),
                         ("few", traces.chunks(lengths, sizes=(2, 3, 2, 64)))):
            _against(run_trace(runner, tr, toks), runs, dtype, f"{kind} {what} {dtype}")


def plain_without_sink(w, config, tokens):
    import plain_ropelix

    keep = plain_ropelix.plain_weights_of
    plain_ropelix.plain_weights_of = lambda s, v, plus_one=False: keep(s, v, False)
    try:
        return plain_forward(w, config, tokens)
    finally:
        plain_ropelix.plain_weights_of = keep


def test_greedy_generation_through_the_engine(cases):
    from fastgen_amd.engine import Engine
    from fastgen_amd.sampling import SamplingParams

    config, weights, folder, toks, _ = cases["trio"]
    prompts = [toks["b"], toks["f"], toks["c"], toks["e"][:40], toks["d"]]
    want = [plain_greedy(weights, config, p, 9) for p in prompts]
    engine = Engine.from_folder(folder, torch.float32, DEV, page_size=16, max_tokens=320, max_batch=3, max_step_tokens=24)
    assert engine.generate(prompts, SamplingParams(temperature=0.0, max_new_tokens=9)) == want
    low = Engine.from_folder(folder, torch.bfloat16, DEV, page_size=64, max_tokens=320, max_batch=3, max_step_tokens=24)
    got = low.generate(prompts, SamplingParams(temperature=0.0, max_new_tokens=9))
    assert [len(g) for g in got] == [9] * len(prompts)


def test_command_lines(cases, tmp_path):
    """The trace runner and the chat tool take the model by its folder, as they take any other."""
    import json
    import subprocess
    import sys
    from pathlib import Path

    import numpy as np

    config, weights, folder, toks, runs = cases["odd"]
    want = runs[torch.float32]["b"]
    root = Path(__file__).resolve().parents[1]
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": toks["b"][:20], "want": [19]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": toks["b"][20:], "want": [0, 16]}], "end": ["x"]}]
    out = tmp_path / "out"
    run = subprocess.run([sys.executable, str(root / "bin" / "trace_run"), "--model", str(folder), "--dtype", "float32",
                          "--out", str(out), "--max-tokens", "64"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                         capture_output=True, text=True, timeout=600)
    assert run.returncode == 0, run.stderr[-2000:]
    assert [l for l in run.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1"]
    got = np.fromfile(out / "1.f32", dtype="<f4").reshape(2, -1)
    assert np.abs(got - want[[20, 36]].numpy()).max() <= 3e-5 * float(want.abs().max())
    chat = subprocess.run([sys.executable, str(root / "bin" / "fgchat"), str(folder), "--prompt-ids", "1,2,3", "--max-tokens",
                           "5", "--temperature", "0"], capture_output=True, text=True, timeout=600)
    assert chat.returncode == 0, chat.stderr[-2000:]
