"""Poselorn on the GPU against the plain implementation (``tests/plain_poselorn.py``) and the kernels' plain twins: each new
kernel alone, then whole models of several shapes under every way of cutting requests into steps, with small pools so
that pages and slots change hands, in float32 (strict) and bfloat16."""

from __future__ import annotations

import copy
from typing import Dict, List

import pytest
import torch

import traces
from helpers import assert_close, make_runner, run_trace, save_model_folder
from plain_poselorn import ODD, ONLY_DELTA, ONLY_LEFT, QUARTET, WIDE, plain_forward, plain_greedy, plain_weights

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
CONFIGS = {"quartet": QUARTET, "odd": ODD, "wide": WIDE, "only_left": ONLY_LEFT, "only_delta": ONLY_DELTA}


def _tokens(config, lengths: Dict[str, int], seed: int) -> Dict[str, List[int]]:
    g = torch.Generator().manual_seed(seed)
    return {r: torch.randint(0, config["vocab"], (n,), generator=g).tolist() for r, n in lengths.items()}


def _close(got, want, dtype, what="", scale=1.0):
    tol = dict(rtol=2e-5, atol=2e-5 * scale) if dtype == torch.float32 else dict(rtol=2e-2, atol=2e-2 * scale)
    torch.testing.assert_close(got.float().cpu(), want.float().cpu(), msg=lambda m: f"{what}: {m}", **tol)


def _dev(x):
    return x.to(DEV).contiguous() if x is not None else None


# ------------------------------------------------------------------ kernels alone
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,D", [(5, 42), (7, 200), (3, 2304), (4, 4096), (2, 8200), (2, 3001)])
def test_terms_added_and_normed(dtype, T, D):
    from fastgen_amd.kernels import ops, twins

    g = torch.Generator().manual_seed(T + D)
    r = lambda *s: torch.randn(*s, generator=g)
    h, again, w1, w2 = r(T, D), r(T, D), torch.rand(D, generator=g) + 0.5, r(D)
    rows = torch.tensor([T - 1, 0, T - 1], dtype=torch.int32)
    term = lambda rows, *more: (rows, *more)
    cases = [[], [term(r(T, D).to(dtype))], [term(r(3, T, D), r(D), r(D))],
             [term(r(T, D).to(dtype), r(D), None, 1e-3), term(r(9, T, D), r(D), r(D), 1e-5), term(r(1, T, D), r(D))],
             [term(r(T, D).to(dtype), None, r(D), 1e-2), term(r(T, D).to(dtype), r(D))]]
    for parts in cases:
        cpu = ops.StreamTerms([ops.StreamTerm(*p) for p in parts])
        gpu = ops.StreamTerms([ops.StreamTerm(*[_dev(x) if isinstance(x, torch.Tensor) else x for x in p]) for p in parts])
        for plus in (None, again):
            hc, hg = h.clone(), _dev(h)
            make = lambda dev, n: [torch.zeros(n, D, dtype=dtype, device=dev) for _ in range(2)]
            gc, gg = make("cpu", 3), make(DEV, 3)
            twins.stream_terms(hc, cpu, plus, [(w1, gc[0])], 1e-5, rows)
            ops.stream_terms(hg, gpu, _dev(plus), [(_dev(w1), gg[0])], 1e-5, _dev(rows))
            assert torch.equal(hg.cpu(), h)
            _close(gg[0], gc[0], dtype, "gathered")
            oc, og = make("cpu", T), make(DEV, T)
            twins.stream_terms(hc, cpu, plus, [(w1, oc[0]), (w2, oc[1])], 1e-5)
            ops.stream_terms(hg, gpu, _dev(plus), [(_dev(w1), og[0]), (_dev(w2), og[1])], 1e-5)
            _close(hg, hc, torch.float32, "stream", 4.0)
            _close(og[0], oc[0], dtype, "first norm")
            _close(og[1], oc[1], dtype, "second norm")
            hg = _dev(h)
            ops.stream_terms(hg, gpu, _dev(plus))
            _close(hg, hc, torch.float32, "stream alone", 4.0)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T", [1, 16, 70, 300])
@pytest.mark.parametrize("K1,N1,per,K2,N2", [(24, 96, 48, 8, 40), (128, 256, 64, 128, 130), (256, 50, 7, 200, 64), (13, 20, 10, 5, 6), (264, 64, 64, 16, 16)])
def test_projections_through_a_narrow_middle(dtype, T, K1, N1, per, K2, N2):
    from fastgen_amd.kernels import ops, twins

    g = torch.Generator().manual_seed(K1 + T)
    src = torch.randn(T, 16 + -(-(K1 + K2) // 8) * 8 + 16, generator=g).to(dtype).float()  # (only the matrix cores round the middle)
    w1, w2 = torch.randn(N1, K1, generator=g).to(dtype), torch.randn(N2, K2, generator=g).to(dtype)
    bias, rate = torch.randn(N1, generator=g), torch.rand(-(-N1 // per), generator=g) + 0.5
    res = []
    for dev, fn in (("cpu", twins), (DEV, ops)):
        o1, o2 = torch.zeros(T, N1 + 4, device=dev)[:, 4:], torch.zeros(T, N2, device=dev)
        to = lambda x: x.to(dev)
        fn.low_rank(to(src), [ops.LowRankJob(8, to(w1), o1, to(bias), to(rate), per), ops.LowRankJob(16 + -(-K1 // 8) * 8, to(w2), o2)])
        res.append((o1, o2))
    for a, b, what in zip(res[1], res[0], ("decays", "products")):
        torch.testing.assert_close(a.cpu(), b, rtol=3e-5, atol=3e-4, msg=lambda m: f"{what}: {m}")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_norms_gates_and_activations(dtype):
    from fastgen_amd.kernels import ops, twins

    g = torch.Generator().manual_seed(3)
    for T, W in ((3, 42), (5, 640), (2, 2050), (3, 4096), (2, 9000)):
        x, w, gate = torch.randn(T, W, generator=g), torch.rand(W, generator=g), torch.randn(T, W + 9, generator=g)
        oc, og = torch.zeros(T, W + 2, dtype=dtype), torch.zeros(T, W + 2, dtype=dtype, device=DEV)
        twins.row_norm_gate(x, w, 1e-5, gate, oc, 0.5)
        ops.row_norm_gate(_dev(x), _dev(w), 1e-5, _dev(gate), og, 0.5)
        _close(og, oc, dtype, f"row norm {W}")
    for H, e in ((3, 14), (4, 128)):
        x, w, gate = torch.randn(6, H * e, generator=g), torch.rand(e, generator=g), torch.randn(6, H * e, generator=g)
        for sigmoid in (False, True):
            oc, og = torch.zeros(6, H * e, dtype=dtype), torch.zeros(6, H * e, dtype=dtype, device=DEV)
            twins.head_norm_gate(x, w, 1e-5, gate, H, oc, 1.0, sigmoid)
            ops.head_norm_gate(_dev(x), _dev(w), 1e-5, _dev(gate), H, og, 1.0, sigmoid)
            _close(og, oc, dtype, f"head norm {H} {sigmoid}")
    for act in ("relu2", "relu", "silu", "gelu_tanh"):
        for N in (40, 2056, 4096):
            x, b = torch.randn(5, N, generator=g), torch.randn(N, generator=g)
            for src, bias in ((x, b), (x.to(dtype), None)):
                _close(ops.bias_act(_dev(src), _dev(bias), act, dtype), twins.bias_act(src, bias, act, dtype), dtype, f"{act} {N}")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,D,E,I,top,groups,keep,ff", [(9, 32, 5, 3, 3, 4, 2, 16), (1, 48, 12, 0, 4, 3, 1, 24), (70, 64, 3, 5, 2, 1, 1, 32),
                                                        (300, 64, 14, 2, 5, 2, 1, 64), (40, 36, 1, 3, 2, 1, 1, 12)])
def test_experts_with_identities(dtype, T, D, E, I, top, groups, keep, ff):
    """Route, sort, both products and the sum against the twins; what no tile writes holds NaN."""
    from fastgen_amd.config import PartSpec
    from fastgen_amd.kernels import ops, twins
    from fastgen_amd.parts import build_part

    part = build_part("feed_forward", PartSpec("moe", "f", dict(
        dim=D, hidden_dim=ff, n_experts=E, identity=I, top=top, router_bias=False, scoring="softmax_all", correction=True,
        n_groups=groups, keep_groups=keep, group_rank="max", renormalize=False)))
    g = torch.Generator().manual_seed(T)
    tensors = {s.name: (torch.randn(s.shape, generator=g) * (s.shape[-1] ** -0.5 if len(s.shape) == 2 else 0.1) - (0.2 if len(s.shape) == 1 else 0.0))
               for s in part.tensor_specs()}
    part.load(tensors, dtype, DEV)
    x = torch.randn(T, D, generator=g).to(dtype)
    route = dict(top=top, correction=tensors["f.correction"], n_groups=groups, keep_groups=keep, softmax_scores=True, group_max=True, raw_weights=True)
    choice, weight = twins.moe_route(x, tensors["f.router.weight"], None, **route)
    cd, wd = ops.moe_route(_dev(x), part.router, None, **{k: _dev(v) if isinstance(v, torch.Tensor) else v for k, v in route.items()})
    assert torch.equal(cd.cpu(), choice)
    _close(wd, weight, torch.float32, "weights")
    sorted_, tiles = ops.moe_sort(cd, E + I, 16, I)
    assert sorted(sorted_.tolist()) == list(range(T * top))
    assert sum(n for _, _, n, _ in tiles.tolist()) == int((choice < E).sum()) and all(e < E for e, _, n, _ in tiles.tolist() if n)
    y = torch.randn(T * top, D, generator=g)
    y[choice.reshape(-1) >= E] = float("nan")
    _close(ops.moe_combine(_dev(y), wd, None, None, cd, E, _dev(x)), twins.moe_combine(y, weight, None, None, choice, E, x), torch.float32, "sum", 4.0)
    low = {k: v.to(dtype).float() for k, v in tensors.items()}
    want = torch.zeros(T, D)
    for t in range(T):
        for j in range(top):
            e = int(choice[t, j])
            out = x[t].float()
            if e < E:
                z = low[f"f.experts.{e}.gate_proj.weight"] @ out
                out = low[f"f.experts.{e}.down_proj.weight"] @ (z * torch.sigmoid(z) * (low[f"f.experts.{e}.up_proj.weight"] @ out)).to(dtype).float()
            want[t] += weight[t, j] * out
    _close(part.forward(_dev(x))[0], want, dtype, "the whole part")


def _conv_inputs(C, K, lens, moves, seed, device="cpu", slots=8):
    from fastgen_amd.kernels import ops

    g = torch.Generator().manual_seed(seed)
    B = len(lens)
    q_start = torch.tensor([0] + torch.tensor(lens).cumsum(0).tolist(), dtype=torch.int32)
    seq = torch.repeat_interleave(torch.arange(B), torch.tensor(lens)).to(torch.int32)
    slot_ids = torch.randperm(slots, generator=g)[:B].to(torch.int32)
    to = lambda x: x.to(device).contiguous()
    return ops.ConvInputs(to(torch.randn(C, K, generator=g)), to(torch.randn(slots, C, max(1, K - 1), generator=g)), 0, to(slot_ids), to(seq),
                          to(q_start), moves)


@pytest.mark.parametrize("lens", [(200, 1, 70), (64, 65), (63, 5, 1), (1, 1, 1, 1), (131,)])
@pytest.mark.parametrize("G,d,H,e,K", [(2, 16, 4, 24, 3), (1, 64, 3, 32, 4), (3, 10, 6, 14, 2), (2, 128, 2, 128, 2), (1, 48, 1, 16, 1),
                                       (1, 272, 2, 20, 2), (2, 208, 2, 40, 2)])
@pytest.mark.parametrize("fading", ["slow", "mixed", "fast"])
def test_delta_rule_with_a_decay_per_channel(lens, G, d, H, e, K, fading):
    """Preparation, and the scan against its twin run in float64, token by token and (with the lengths on the host) in
    chunks.  Decays reach from a state that never fades to channels forgotten within a token: the sums inside 16 tokens as
    products and pair by pair, side by side in one call."""
    from fastgen_amd.kernels import ops, twins

    C, T, B = 2 * G * d + H * e, sum(lens), len(lens)
    g = torch.Generator().manual_seed(d + T)
    src = torch.randn(T, C + H + 3, generator=g)
    moves = max(lens) == 1
    col = -(-(C + H) // 4) * 4
    width = -(-(col + H * d) // 4) * 4
    cc, cg = _conv_inputs(C, K, lens, moves, 7), _conv_inputs(C, K, lens, moves, 7, DEV)
    rc, rg = torch.zeros(T, width), torch.zeros(T, width, device=DEV)
    twins.delta_prepare(src, G, d, H, e, cc, C, -1, None, None, d ** -0.5, 1e-6, rc)
    ops.delta_prepare(_dev(src), G, d, H, e, cg, C, -1, None, None, d ** -0.5, 1e-6, rg)
    _close(rg, rc, torch.float32, "prepared rows", 4.0)
    log_g = -torch.rand(T, H * d, generator=g) * {"slow": 0.02, "mixed": 1.0, "fast": 3.0}[fading]
    if fading != "slow":
        log_g[:, ::5] *= 1e-3
    if fading == "mixed":  # some channels of some tokens are gone at once
        log_g[torch.rand(T, H * d, generator=g) < 0.02] = -200.0
    if fading == "fast":
        log_g[:, 1::7] = -30.0
    rc[:, col : col + H * d] = log_g
    state = torch.randn(8, H * d * e + 6, generator=g)  # (slots with a stride of their own)
    view = lambda s: s[:, : H * d * e].view(8, H, d, e)
    sc, oc = state.double(), torch.empty(T, H * e, dtype=torch.float64)
    twins.delta_scan(rc.double(), G, d, H, e, view(sc), cc.slot_ids, cc.q_start, B, oc, None, col)
    for host in (None, cc.q_start.numpy()):
        sg, og = _dev(state), torch.full((T, H * e), float("nan"), device=DEV)
        ops.delta_scan(_dev(rc), G, d, H, e, view(sg), cg.slot_ids, cg.q_start, B, og, host, col)
        what = "token by token" if host is None else "chunks"
        assert float((og.double().cpu() - oc).abs().max()) <= 2e-5 * max(1.0, float(oc.abs().max())), what
        assert float((sg.double().cpu() - sc).abs().max()) <= 2e-5 * max(1.0, float(sc.abs().max())), f"{what}: state"


@pytest.mark.parametrize("lens", [(200, 1, 70), (64, 65), (63, 5, 1), (1, 1, 1, 1), (700,)])
@pytest.mark.parametrize("H,d,e", [(3, 16, 24), (2, 64, 32), (6, 10, 14), (2, 128, 128), (1, 48, 300), (2, 272, 20), (2, 192, 40), (5, 7, 9)])
def test_linear_attention_with_constant_decays(lens, H, d, e):
    """The scan against its twin run in float64, token by token and in chunks; decays from none at all to a state that keeps
    nothing."""
    from fastgen_amd.kernels import ops, twins

    T, B = sum(lens), len(lens)
    g = torch.Generator().manual_seed(d + T)
    rows = torch.randn(T, -(-(2 * H * d + H * e) // 4) * 4 + 4, generator=g)
    log_decay = torch.log(torch.tensor([0.9995, 1.0, 0.3, 0.97, 0.8, 0.9][:H]))
    if H == 6:
        log_decay[5] = -1e4
    q_start = torch.tensor([0] + torch.tensor(lens).cumsum(0).tolist(), dtype=torch.int32)
    slots = torch.randperm(8, generator=g)[:B].to(torch.int32)
    state = torch.randn(8, H, d, e, generator=g)
    sc, oc = state.double(), torch.empty(T, H * e, dtype=torch.float64)
    cols = (0, H * d, 2 * H * d)
    twins.lightning_scan(rows.double(), *cols, log_decay, sc, slots, q_start, B, oc)
    for host in (None, q_start.numpy()):
        sg, og = _dev(state), torch.full((T, H * e), float("nan"), device=DEV)
        ops.lightning_scan(_dev(rows), *cols, _dev(log_decay), sg, _dev(slots), _dev(q_start), B, og, host)
        what = "token by token" if host is None else "chunks"
        tol = 1e-4 if host is None and T >= 500 else 2e-5  # (a decay rounded to fp32, hundreds of times over)
        assert float((og.double().cpu() - oc).abs().max()) <= tol * max(1.0, float(oc.abs().max())), what
        assert float((sg.double().cpu() - sc).abs().max()) <= tol * max(1.0, float(sc.abs().max())), f"{what}: state"


# ----------------------------------------------------------------- whole models
LENGTHS = {"a": 150, "b": 37, "c": 2, "d": 1, "e": 70, "f": 19}


# Whole models are compared in float32 with routers that choose token by token, and in bfloat16 with corrections that decide
# the choice alone: a choice between two near scores may fall either way under bfloat16's rounding, and a token that goes
# to another expert is far off without a fault.  (The routed part's own test above chooses token by token in both.)
DTYPES = (torch.float32, torch.bfloat16)


def _weights(config, seed, dtype):
    return plain_weights(config, seed, decisive=dtype == torch.bfloat16)


def _runs(weights, config, toks, dtype):
    return {dt: {r: plain_forward(weights, config, t, dt) for r, t in toks.items()} for dt in (torch.float64, dtype)}


@pytest.fixture(scope="module")
def cases(tmp_path_factory):
    """By (configuration's name, dtype): configuration, weights, folder, tokens, plain runs."""
    out = {}
    for name, config in CONFIGS.items():
        toks = _tokens(config, LENGTHS, seed=7)
        for dtype in DTYPES:
            weights = _weights(config, len(name), dtype)
            folder = save_model_folder(tmp_path_factory.mktemp(name), config, weights)
            out[name, dtype] = (config, weights, folder, toks, _runs(weights, config, toks, dtype))
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
    config, weights, folder, toks, runs = cases[name, torch.float32]
    runner = make_runner(folder, torch.float32, page_size=16, max_tokens=304, max_requests=4)
    first = None
    for kind, tr in _all_traces(LENGTHS).items():
        got = run_trace(runner, tr, toks)
        _against(got, runs, torch.float32, f"poselorn {name} {kind}")
        if first is None:
            first = got
        for r in got:
            assert float((got[r] - first[r]).abs().max()) <= 1e-5 * float(first[r].abs().max()), f"{name} {kind}: {r} depends on the cut"
        assert all(runner.cache.free_pages(g) == 304 // 16 for g in range(runner.cache.n_groups))
        assert runner.cache.free_slots() == 4


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_bfloat16_every_cut_batch_and_reuse(cases, name):
    config, weights, folder, toks, runs = cases[name, torch.bfloat16]
    for page, pool in ((16, 304), (64, 768)):
        runner = make_runner(folder, torch.bfloat16, page_size=page, max_tokens=pool, max_requests=4)
        for kind, tr in _all_traces(LENGTHS).items():
            _against(run_trace(runner, tr, toks), runs, torch.bfloat16, f"poselorn {name} {kind} bfloat16, pages of {page}")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_the_stream_after_every_layer(cases, dtype):
    from fastgen_amd.engine import Model, ModelRunner, StepEntry
    from fastgen_amd.kernels import ops

    config, weights, folder, toks, _ = cases["quartet", dtype]
    want: list = []
    plain_forward(weights, config, toks["b"], dtype, want)
    model = Model.from_folder(folder, dtype, DEV)
    seen = []
    for block in model.parts.blocks:
        def wrap(keep=block.forward):
            def forward(h, pending, ctx, store):
                out = keep(h, pending, ctx, store)
                after = h.clone()
                ops.stream_terms(after, out)
                seen.append(after.cpu())
                return out
            return forward
        block.forward = wrap()
    runner = ModelRunner(model, page_size=16, max_tokens=64, max_requests=1)
    runner.step([StepEntry("b", toks["b"], [0])])
    assert len(seen) == len(want) == 8
    for i, (g, w) in enumerate(zip(seen, want)):
        tol = 2e-5 if dtype == torch.float32 else 4e-2
        assert float((g - w.float()).abs().max()) <= tol * float(w.abs().max()), f"after layer run {i}"


@pytest.mark.parametrize("name", ["quartet", "odd"])
def test_long_decoding_across_pages_and_windows(cases, name):
    """A short prompt, then 290 tokens one by one over many pages and past every window (recorded steps)."""
    for dtype, page in ((torch.float32, 16), (torch.bfloat16, 16), (torch.bfloat16, 64)):
        config, weights, folder, _, _ = cases[name, dtype]
        toks = _tokens(config, {"z": 300}, seed=5)
        runs = _runs(weights, config, toks, dtype)
        runner = make_runner(folder, dtype, page_size=page, max_tokens=320, max_requests=2)
        _against(run_trace(runner, traces.tail({"z": 300}, 290), toks), runs, dtype, f"poselorn {name} long decoding {dtype}")


@pytest.mark.parametrize("name", ["quartet", "wide"])
def test_long_prompts_beside_short_ones(cases, name):
    """Prompts of several hundred tokens in one step (recurrences in chunks), together in one batch, in two steps and in
    small portions."""
    lengths = {"p": 500, "q": 260, "r": 3}
    together = [([("p", 0, 500), ("q", 0, 260), ("r", 0, 3)], ["p", "q", "r"])]
    for dtype, page in ((torch.float32, 16), (torch.bfloat16, 64)):
        config, weights, folder, _, _ = cases[name, dtype]
        toks = _tokens(config, lengths, seed=13)
        runs = _runs(weights, config, toks, dtype)
        runner = make_runner(folder, dtype, page_size=page, max_tokens=896, max_requests=3)
        for kind, tr in (("whole", traces.whole(lengths)), ("together", together),
                         ("halves", traces.chunks(lengths, sizes=(290, 210))), ("portions", traces.chunks(lengths))):
            _against(run_trace(runner, tr, toks), runs, dtype, f"poselorn {name} long {kind} {dtype}")


def test_many_sequences_decoding_together(cases):
    """Twenty requests decode side by side: recorded steps filled up with stand-in sequences, whose state is nobody's."""
    prompts = {f"s{i}": 3 + 5 * (i % 7) for i in range(20)}
    lengths = {r: n + 12 for r, n in prompts.items()}
    tr = traces.many_decoding_together(prompts, 12, seed=1)
    for dtype in DTYPES:
        config, weights, folder, _, _ = cases["quartet", dtype]
        toks = _tokens(config, lengths, seed=3)
        runs = _runs(weights, config, toks, dtype)
        runner = make_runner(folder, dtype, page_size=64, max_tokens=64 * 20, max_requests=20)
        _against(run_trace(runner, tr, toks), runs, dtype, f"poselorn many decoding {dtype}")


@pytest.mark.parametrize("window", [32, 21, 16, 1])
def test_keys_at_the_edges_of_windows_and_pages(tmp_path, window):
    """One attention layer with sharp scores and windows at and off a page's border: the plain run with a window one token
    longer or shorter differs by far more than the tolerance, and the engine agrees with the right one, for whole prompts,
    portions down to two tokens and tokens decoded alone."""
    n = 130
    config = copy.deepcopy(ONLY_LEFT)
    at = config["layers"][0]["mixer"]["left"]
    at["mask"]["size"], at["scale"] = window, 3 * at["scale"]
    w = plain_weights(config, window)
    toks = _tokens(config, {"s": n}, seed=window)
    runs = {dt: _runs(w, config, toks, dt) for dt in DTYPES}
    want = runs[torch.float32][torch.float32]["s"]
    for other_size in {max(1, window - 1), window + 1} - {window}:
        other = copy.deepcopy(config)
        other["layers"][0]["mixer"]["left"]["mask"]["size"] = other_size
        moved = (plain_forward(w, other, toks["s"]) - want).abs().amax(-1)
        assert float(moved[window:].max()) > 0.05 * float(want.abs().max()), "the window's edge does not decide"
    folder = save_model_folder(tmp_path / str(window), config, w)
    for dtype, page in ((torch.float32, 16), (torch.bfloat16, 16), (torch.bfloat16, 64)):
        runner = make_runner(folder, dtype, page_size=page, max_tokens=192, max_requests=1)
        for kind, tr in (("whole", traces.whole({"s": n})), ("tail", traces.tail({"s": n}, 90)), ("chunks", traces.chunks({"s": n})),
                         ("pairs", traces.chunks({"s": n}, sizes=(2, 3, 2, 5)))):
            _against(run_trace(runner, tr, toks), runs[dtype], dtype, f"window {window} {kind} {dtype}")


@pytest.mark.parametrize("kind", ["delta", "right"])
def test_a_state_that_remembers(tmp_path, kind):
    """Recurrences that hardly forget: changing the first 40 tokens of hundreds changes the last logits, whole, in portions,
    decoded alone, through slots that another request held."""
    config = copy.deepcopy({"delta": ONLY_DELTA, "right": ONLY_LEFT}[kind])
    m, n = config["layers"][0]["mixer"], {"delta": 200, "right": 400}[kind]
    if kind == "delta":  # (keys of 64: a later write leaves most of an earlier one standing)
        m.update(dim=64)
    else:
        m["left"]["mask"]["size"] = 4
        m["right"].update(heads=2, dim=16, vdim=16, decay=[0.9995, 1.0])
    w = plain_weights(config, 9)
    if kind == "delta":
        w["l0.mix.A_log"].fill_(-9.0)
    lengths = {"other": 70, "s": n}
    toks = _tokens(config, lengths, seed=2)
    runs = {dt: _runs(w, config, toks, dt) for dt in DTYPES}
    want = runs[torch.float32][torch.float32]["s"]
    changed = [(t + 1) % config["vocab"] if i < 40 else t for i, t in enumerate(toks["s"])]
    assert float((plain_forward(w, config, changed)[-30:] - want[-30:]).abs().max()) > 0.01 * float(want.abs().max()), "nothing is remembered"
    folder = save_model_folder(tmp_path / kind, config, w)
    for dtype, page in ((torch.float32, 16), (torch.bfloat16, 64)):
        runner = make_runner(folder, dtype, page_size=page, max_tokens=448, max_requests=1)
        for what, tr in (("whole", traces.whole(lengths)), ("tail", traces.tail(lengths, 40)), ("chunks", traces.chunks(lengths)),
                         ("few", traces.chunks(lengths, sizes=(2, 3, 2, 64)))):
            _against(run_trace(runner, tr, toks), runs[dtype], dtype, f"{kind} {what} {dtype}")


def test_greedy_generation_through_the_engine(cases):
    from fastgen_amd.engine import Engine
    from fastgen_amd.sampling import SamplingParams

    config, weights, folder, toks, _ = cases["quartet", torch.float32]
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

    config, weights, folder, toks, runs = cases["odd", torch.float32]
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
