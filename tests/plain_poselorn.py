"""A plain, slow Poselorn: whole sequences, no cache, no batching, one function
per mechanism, sharing no code with ``fastgen_amd``.  It is what the engine is
compared with.

The model (notation of this file).  ``x = E[token] * s``; a layer adds both of its sublayers at once,

    x <- x + c * (ls1 (.) mixer(n1(x)) + ls2 (.) ff(n2(x)))

with ``n(x) = x / rms(x) * w``, one number ``c`` for the model and a vector ``ls`` for each sublayer.  A stretch of layers
may run several times; every pass but the first starts from ``x + x0``, ``x0`` the embedding's output.  The logits are
``W n(x)``.  Two mixers exist:

* ``channel_delta``: the delta rule with a decay per key channel.  q, k, v pass a causal convolution and silu, q and k
  become unit vectors; ``S <- diag(g) S;  S <- S + k (b (v - S^T k))^T;  o = S^T q``, a norm per head, times the sigmoid of a
  projection through a narrow middle.
* ``parallel``: half the sum of two normed outputs.  *left* is softmax attention of grouped heads in a sliding window, q, k, v
  with biases, a norm per head on q and k, rotated pairs ``(i, i + n/2)``.  *right* is linear attention with a constant
  decay per head, ``S <- a S + k v^T;  o = S^T q`` with silu on q, k and v, one norm over all heads, a sigmoid gate.

The feed-forward is ``W_down relu(W_up h + b)^2 + b'`` or a mixture of gated experts, some of which return their input.

``dtype`` is the precision of matrix products and activations; the stream, norms, angles, scores, weights, the router and
everything inside a recurrence stay in float32 (float64 when the whole run is).
"""

from __future__ import annotations

import math
from typing import Dict, List, Mapping, Optional, Tuple

import torch


def _hi(x: torch.Tensor) -> torch.Tensor:
    return x if x.dtype == torch.float64 else x.float()


def _mm(x: torch.Tensor, w: torch.Tensor, dtype: torch.dtype, bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``x W^T + b`` with operands in ``dtype``, summed in the high precision, rounded once to ``dtype``."""
    y = _hi(x.to(dtype)) @ _hi(w.to(dtype)).T
    return (y if bias is None else y + _hi(bias)).to(dtype)


# ------------------------------------------------------------------ mechanisms
def plain_rms(x: torch.Tensor, w: Optional[torch.Tensor], eps: float) -> torch.Tensor:
    x = _hi(x)
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if w is None else y * _hi(w)


def plain_silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def plain_unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def plain_rotate(x: torch.Tensor, base: float, dims: int) -> torch.Tensor:
    """``x [T, heads, d]``: pairs ``(i, i + dims/2)`` of a head's first ``dims`` turn by ``p * base^(-2i/dims)``."""
    x = _hi(x).clone()
    half = dims // 2
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=x.dtype)
    ang = torch.arange(x.shape[0], dtype=x.dtype)[:, None] * f[None, :]
    cos, sin = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    u, v = x[..., :half].clone(), x[..., half:dims].clone()
    x[..., :half] = u * cos - v * sin
    x[..., half:dims] = v * cos + u * sin
    return x


def plain_window(T: int, size: Optional[int]) -> torch.Tensor:
    """``[query, key]``: the query's own token and the ``size - 1`` before it (all of them without a size)."""
    i = torch.arange(T)
    n = i[:, None] - i[None, :]
    return (n >= 0) & (n < size) if size else n >= 0


def plain_window_attention(q, k, v, scale: float, size: Optional[int]) -> torch.Tensor:
    """``q [T, H, d]``, ``k [T, G, d]``, ``v [T, G, e]`` -> ``[T, H * e]``: plain softmax over the window."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    seen, out = plain_window(T, size), []
    for h in range(H):
        s = _hi(q[:, h]) @ _hi(k[:, h // (H // G)]).T * scale
        out.append(torch.softmax(s.masked_fill(~seen, -math.inf), -1) @ _hi(v[:, h // (H // G)]))
    return torch.stack(out, 1).reshape(T, -1)


def plain_conv(u: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """``y_t[c] = sum_j taps[c, j] u_(t - K + 1 + j)[c]``, zeros before the start."""
    u, taps = _hi(u), _hi(taps)
    K = taps.shape[1]
    pad = torch.cat([u.new_zeros(K - 1, u.shape[1]), u])
    return sum(pad[j : j + u.shape[0]] * taps[:, j].to(u.dtype) for j in range(K))


def plain_channel_delta(q, k, v, g, beta) -> torch.Tensor:
    """One head: ``q, k, g [T, d]``, ``v [T, e]``, ``beta [T]`` -> ``o [T, e]``; a row of the state fades by its own ``g``."""
    S, out = q.new_zeros(q.shape[1], v.shape[1]), []
    for t in range(q.shape[0]):
        S = g[t][:, None] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + k[t][:, None] * u[None, :]
        out.append(S.T @ q[t])
    return torch.stack(out)


def plain_decayed_attention(q, k, v, decay: float) -> torch.Tensor:
    """One head: ``S <- decay S + k v^T``, ``o = S^T q``."""
    S, out = q.new_zeros(q.shape[1], v.shape[1]), []
    for t in range(q.shape[0]):
        S = decay * S + k[t][:, None] * v[t][None, :]
        out.append(S.T @ q[t])
    return torch.stack(out)


def plain_delta_mixer(x, w: Mapping[str, torch.Tensor], p: str, m: Mapping, eps: float, dtype: torch.dtype) -> torch.Tensor:
    T, H, G, d, e = x.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    conv = lambda n: _hi(plain_silu(plain_conv(_mm(x, w[f"{p}.{n}"], dtype), w[f"{p}.{n}.conv"])).to(dtype))
    q = plain_unit(conv("q").view(T, G, d)) * d ** -0.5
    k = plain_unit(conv("k").view(T, G, d))
    v = conv("v").view(T, H, e)
    narrow = lambda n: _hi(_mm(x, w[f"{p}.{n}1"], dtype)) @ _hi(w[f"{p}.{n}2"]).T
    beta = torch.sigmoid(_hi(x.to(dtype)) @ _hi(w[f"{p}.b"]).T)
    step = torch.nn.functional.softplus(narrow("a") + _hi(w[f"{p}.dt_bias"])).view(T, H, d)
    g = torch.exp(-torch.exp(_hi(w[f"{p}.A_log"]))[:, None] * step)
    o = torch.stack([plain_channel_delta(q[:, h // (H // G)], k[:, h // (H // G)], v[:, h], g[:, h], beta[:, h])
                     for h in range(H)], dim=1)
    o = plain_rms(o, w[f"{p}.norm"], eps) * torch.sigmoid(narrow("g")).view(T, H, e)
    return _mm(o.reshape(T, H * e).to(dtype), w[f"{p}.o"], dtype)


def plain_left(x, w: Mapping[str, torch.Tensor], p: str, m: Mapping, eps: float, dtype: torch.dtype) -> torch.Tensor:
    T, H, G, d, e = x.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = plain_rms(_mm(x, w[f"{p}.q"], dtype, w[f"{p}.q.b"]).view(T, H, d), w[f"{p}.q.norm"], eps)
    k = plain_rms(_mm(x, w[f"{p}.k"], dtype, w[f"{p}.k.b"]).view(T, G, d), w[f"{p}.k.norm"], eps)
    v = _mm(x, w[f"{p}.v"], dtype, w[f"{p}.v.b"]).view(T, G, e)
    rot = m.get("rot") or {"base": 1.0, "dims": 0}
    q = plain_rotate(q, rot["base"], rot["dims"]).to(dtype)
    k = plain_rotate(k, rot["base"], rot["dims"]).to(dtype)
    o = plain_window_attention(q, k, v, m["scale"], (m.get("mask") or {}).get("size"))
    return _mm(o.to(dtype), w[f"{p}.o"], dtype)


def plain_right(x, w: Mapping[str, torch.Tensor], p: str, m: Mapping, eps: float, dtype: torch.dtype) -> torch.Tensor:
    T, H, d, e = x.shape[0], m["heads"], m["dim"], m["vdim"]
    part = lambda n, wide: plain_silu(_hi(_mm(x, w[f"{p}.{n}"], dtype))).view(T, H, wide)
    q, k, v = part("q", d), part("k", d), part("v", e)
    o = torch.stack([plain_decayed_attention(q[:, h], k[:, h], v[:, h], m["decay"][h]) for h in range(H)], dim=1)
    o = plain_rms(o.reshape(T, H * e), w[f"{p}.norm"], eps) * torch.sigmoid(_hi(_mm(x, w[f"{p}.g"], dtype)))
    return _mm(o.to(dtype), w[f"{p}.o"], dtype)


def plain_mixer(h, w, p: str, kind: str, m: Mapping, eps: float, dtype: torch.dtype) -> torch.Tensor:
    if kind == "parallel":
        left = plain_rms(plain_left(h, w, f"{p}.left", m["left"], eps, dtype), w[f"{p}.left.out"], eps)
        right = plain_rms(plain_right(h, w, f"{p}.right", m["right"], eps, dtype), w[f"{p}.right.out"], eps)
        return 0.5 * (left + right)
    if kind == "channel_delta":
        return _hi(plain_delta_mixer(h, w, p, m, eps, dtype))
    raise ValueError(kind)


def plain_dense(h, w, p: str, dtype: torch.dtype) -> torch.Tensor:
    z = torch.relu(_hi(_mm(h, w[f"{p}.up"], dtype, w[f"{p}.up.b"]))) ** 2
    return _hi(_mm(z.to(dtype), w[f"{p}.down"], dtype, w[f"{p}.down.b"]))


def plain_route(z: torch.Tensor, correction: torch.Tensor, top: int, groups: int, keep: int) -> Tuple[List[int], List[float]]:
    """One token's chosen experts and their weights, from its router logits."""
    s = torch.softmax(z, 0)
    c = (s + correction).tolist()
    per = len(c) // groups
    best = sorted(range(groups), key=lambda g: -max(c[g * per : (g + 1) * per]))[:keep]
    may = [i for i in range(len(c)) if i // per in best]
    chosen = sorted(may, key=lambda i: -c[i])[:top]
    return chosen, [float(s[i]) for i in chosen]


def plain_expert(h, w, p: str, dtype: torch.dtype) -> torch.Tensor:
    a = plain_silu(_hi(_mm(h, w[f"{p}.gate"], dtype))) * _hi(_mm(h, w[f"{p}.up"], dtype))
    return _hi(_mm(a.to(dtype), w[f"{p}.down"], dtype))


def plain_experts(h, w, p: str, m: Mapping, dtype: torch.dtype) -> torch.Tensor:
    r = m["router"]
    z = _hi(h) @ _hi(w[f"{p}.router"]).T
    groups = r.get("groups") or {"count": 1, "keep": 1}
    routes = [plain_route(z[t], _hi(w[f"{p}.correction"]), r["top"], groups["count"], groups["keep"]) for t in range(h.shape[0])]
    out = torch.zeros_like(_hi(h))
    for e in range(z.shape[1]):
        rows = [t for t, (chosen, _) in enumerate(routes) if e in chosen]
        if rows:
            weight = torch.tensor([routes[t][1][routes[t][0].index(e)] for t in rows], dtype=out.dtype)
            y = plain_expert(h[rows], w, f"{p}.e{e}", dtype) if e < r["experts"] else _hi(h[rows])
            out[rows] += weight[:, None] * y
    return out


# ----------------------------------------------------------------------- model
def plain_order(config: Mapping) -> List[Tuple[int, bool]]:
    """The layers in the order they run, and whether the embedding's output is added before."""
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    body = [(i, t > 0 and i == a) for t in range(loop["times"]) for i in range(a, b)]
    return [(i, False) for i in range(a)] + body + [(i, False) for i in range(b, n)]


def plain_forward(weights: Mapping[str, torch.Tensor], config: Mapping, tokens: List[int],
                  dtype: torch.dtype = torch.float32, layers_out: Optional[list] = None) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one whole sequence.  ``layers_out``: a list that gets the stream after every layer run."""
    if dtype == torch.float64:
        w = {k: v.double() if v.dtype.is_floating_point else v for k, v in weights.items()}
    else:
        w = {k: v.to(dtype) if v.dtype.is_floating_point else v for k, v in weights.items()}
    eps, mult = config["norm"]["eps"], config["residual_mult"]
    x0 = x = _hi(w["embed"][torch.tensor(tokens)]) * config["embedding"]["scale"]
    for i, again in plain_order(config):
        layer, p = config["layers"][i], f"l{i}"
        if again:
            x = x + x0
        h = plain_rms(x, w[f"{p}.norm1"], eps).to(dtype)
        add = plain_mixer(h, w, f"{p}.mix", layer["type"], layer["mixer"], eps, dtype) * _hi(w[f"{p}.ls1"])
        mlp = layer.get("mlp")
        if mlp is not None:
            h = plain_rms(x, w[f"{p}.norm2"], eps).to(dtype)
            y = plain_dense(h, w, f"{p}.mlp", dtype) if mlp["kind"] == "dense" else plain_experts(h, w, f"{p}.mlp", mlp, dtype)
            add = add + y * _hi(w[f"{p}.ls2"])
        x = x + mult * add
        if layers_out is not None:
            layers_out.append(x)
    h = plain_rms(x, w["final.norm"], eps).to(dtype)
    return _hi(h) @ _hi(w["head"]).T


def plain_greedy(weights: Mapping[str, torch.Tensor], config: Mapping, prompt: List[int], n_new: int,
                 dtype: torch.dtype = torch.float32) -> List[int]:
    """``n_new`` tokens, each the argmax of the last position's logits of the whole sequence so far."""
    seq, out = list(prompt), []
    for _ in range(n_new):
        tok = int(plain_forward(weights, config, seq, dtype)[-1].argmax())
        out.append(tok)
        seq.append(tok)
    return out


# --------------------------------------------------------------------- weights
def plain_weights(config: Mapping, seed: int, stored: torch.dtype = torch.bfloat16, a_rank: int = 6, g_rank: int = 10,
                  decisive: bool = False) -> Dict[str, torch.Tensor]:
    """Random tensors of a configuration, by the names of the checkpoint, with the values that ``stored`` can hold
    (as float32).  ``a_rank`` / ``g_rank``: the narrow middles, which only the tensors' shapes give.
    ``decisive``: corrections so far apart that they alone decide which experts are chosen, whatever the rounding."""
    g = torch.Generator().manual_seed(seed)
    D, V = config["width"], config["vocab"]
    w: Dict[str, torch.Tensor] = {}

    def mat(name, rows, cols, std=None):
        w[name] = torch.randn(rows, cols, generator=g) * (std if std is not None else cols ** -0.5)

    def vec(name, *shape, mean=0.0, std=0.1):
        w[name] = mean + std * torch.randn(*shape, generator=g)

    mat("embed", V, D, 0.5)
    mat("head", V, D, 0.5)
    vec("final.norm", D, mean=1.0)
    for i, layer in enumerate(config["layers"]):
        m, p = layer["mixer"], f"l{i}.mix"
        vec(f"l{i}.norm1", D, mean=1.0)
        vec(f"l{i}.ls1", D, mean=1.0, std=0.2)
        if layer["type"] == "parallel":
            a, r = m["left"], m["right"]
            for n, c in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"])):
                mat(f"{p}.left.{n}", c, D)
                vec(f"{p}.left.{n}.b", c, std=0.3)
            vec(f"{p}.left.q.norm", a["dim"], mean=1.0, std=0.2)
            vec(f"{p}.left.k.norm", a["dim"], mean=1.0, std=0.2)
            mat(f"{p}.left.o", D, a["heads"] * a["vdim"])
            vec(f"{p}.left.out", D, mean=1.0, std=0.2)
            for n, c in (("q", r["dim"]), ("k", r["dim"]), ("v", r["vdim"]), ("g", r["vdim"])):
                mat(f"{p}.right.{n}", r["heads"] * c, D)
            vec(f"{p}.right.norm", r["heads"] * r["vdim"], mean=1.0, std=0.2)
            mat(f"{p}.right.o", D, r["heads"] * r["vdim"])
            vec(f"{p}.right.out", D, mean=1.0, std=0.2)
        else:
            H, G, d, e, K = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
            for n, c in (("q", G * d), ("k", G * d), ("v", H * e)):
                mat(f"{p}.{n}", c, D)
                vec(f"{p}.{n}.conv", c, K, std=0.6)
            mat(f"{p}.b", H, D)
            vec(f"{p}.A_log", H, mean=-1.0, std=1.0)
            mat(f"{p}.a1", a_rank, D)
            mat(f"{p}.a2", H * d, a_rank)
            vec(f"{p}.dt_bias", H * d, mean=-2.0, std=1.0)
            mat(f"{p}.g1", g_rank, D)
            mat(f"{p}.g2", H * e, g_rank)
            vec(f"{p}.norm", e, mean=1.0, std=0.2)
            mat(f"{p}.o", D, H * e)
        mlp = layer.get("mlp")
        if mlp is None:
            continue
        vec(f"l{i}.norm2", D, mean=1.0)
        vec(f"l{i}.ls2", D, mean=1.0, std=0.2)
        p = f"l{i}.mlp"
        if mlp["kind"] == "dense":
            mat(f"{p}.up", mlp["ff"], D)
            vec(f"{p}.up.b", mlp["ff"], std=0.3)
            mat(f"{p}.down", D, mlp["ff"])
            vec(f"{p}.down.b", D, std=0.3)
        else:
            r, ff = mlp["router"], mlp["expert"]["ff"]
            n = r["experts"] + r.get("identity", 0)
            mat(f"{p}.router", n, D)
            vec(f"{p}.correction", n, mean=-0.05, std=0.1)
            if decisive:
                w[f"{p}.correction"] = 2.0 * (torch.randperm(n, generator=g) - n // 2)
            for e in range(r["experts"]):
                mat(f"{p}.e{e}.gate", ff, D)
                mat(f"{p}.e{e}.up", ff, D)
                mat(f"{p}.e{e}.down", D, ff, 2 * ff ** -0.5)
    return {k: v.to(stored).float() for k, v in w.items()}


# ---------------------------------------------------------------- configurations
def _delta(heads, kv, dim, vdim, conv):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}


def _parallel(left, right, decay):
    """``left``: heads, kv_heads, dim, vdim, rotated dims, window; ``right``: heads, dim, vdim."""
    heads, kv, dim, vdim, rot, window = left
    l = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": dim ** -0.5}
    if rot:
        l["rot"] = {"base": 900.0, "dims": rot}
    if window:
        l["mask"] = {"size": window}
    return {"left": l, "right": {"heads": right[0], "dim": right[1], "vdim": right[2], "decay": list(decay)}}


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _experts(experts, identity, top, ff, groups=None):
    r = {"experts": experts, "identity": identity, "top": top}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r}


def _model(width, vocab, layers, loop=None, embed=3.0, mult=0.6, eps=1e-5):
    c = {"architecture": "Poselorn", "width": width, "vocab": vocab, "embedding": {"scale": embed}, "residual_mult": mult,
         "norm": {"eps": eps}, "layers": [{"type": t, "mixer": m, "mlp": f} for t, m, f in layers]}
    if loop:
        c["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return c


# both mixers under both feed-forwards and under none; the middle layers run three times
QUARTET = _model(64, 96, [
    ("parallel", _parallel((4, 2, 16, 24, 8, 20), (3, 16, 8), (0.5, 0.93, 0.998)), _dense(56)),
    ("channel_delta", _delta(4, 2, 16, 24, 3), _experts(10, 2, 3, 24, (3, 2))),
    ("parallel", _parallel((4, 1, 16, 16, 16, 32), (2, 24, 16), (0.9, 0.99)), None),
    ("channel_delta", _delta(2, 2, 32, 16, 2), _dense(40))], loop=(1, 3, 3))
# heads that are no power of two, head sizes that are no multiple of 16 (or of 8), values narrower than keys, one head a
# side, no window, nothing rotated, one tap, widths that are no multiple of 8, no identity experts, groups of one, every
# group kept; nothing runs twice
ODD = _model(72, 50, [
    ("channel_delta", _delta(6, 3, 10, 14, 1), _experts(5, 0, 2, 20)),
    ("parallel", _parallel((3, 3, 20, 6, 0, None), (1, 10, 6), (0.97,)), _experts(6, 1, 4, 12, (7, 5))),
    ("parallel", _parallel((5, 5, 12, 12, 4, 7), (5, 6, 14), (0.2, 0.7, 0.9, 0.99, 1.0)), _experts(4, 4, 3, 16, (2, 2))),
    ("channel_delta", _delta(3, 1, 22, 6, 5), None)], embed=1.0, mult=1.0, eps=1e-6)
# more query heads a key head than the matrix-core kernels group; every layer looped; more identity experts than others
WIDE = _model(40, 80, [
    ("parallel", _parallel((20, 1, 8, 8, 8, 16), (4, 8, 32), (0.6, 0.8, 0.95, 0.999)), _experts(3, 5, 2, 16, (4, 1))),
    ("channel_delta", _delta(2, 1, 64, 40, 4), _experts(12, 4, 5, 16, (4, 2)))], loop=(0, 2, 2), embed=2.0)
ONLY_LEFT = _model(48, 64, [("parallel", _parallel((4, 2, 16, 16, 8, 32), (1, 8, 8), (0.5,)), None)], mult=1.0)
ONLY_DELTA = _model(48, 64, [("channel_delta", _delta(4, 2, 16, 16, 4), None)], mult=1.0)
