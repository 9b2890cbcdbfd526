"""A plain, slow Ropelix: whole sequences, no cache, no batching, one function
per mechanism, sharing no code with ``fastgen_amd``.  It is what the engine is
compared with.

The model (notation of this file).  ``x = E[token] * s``; a layer does

    x <- x + m * ls1 (.) mixer(n1(x));   x <- x + m * ls2 (.) ff(n2(x))

with ``n(x) = x / rms(x) * (1 + w)``, one number ``m`` for the model and a vector ``ls`` for each sublayer;
the logits are ``E n(x)``.  Three mixers exist:

* ``parallel``: two mixers read the same rows, ``left_scale * left + right_scale * right``.  *left* is softmax
  attention of grouped heads: one RMS norm over all of a token's query rows and one over all its key rows,
  rotation of the first ``rot`` dimensions of a head (pairs ``i, i + rot/2``), scores through ``cap * tanh(s / cap)``,
  a sliding window, and the heads' weights of a (query, key) pair mixed by a matrix after the softmax.
  *right* is a real-gated linear recurrence: ``u`` (a projection, then a causal convolution) drives
  ``S <- a S + sqrt(1 - a^2) i u`` per channel with ``a = exp(-8 r softplus(lam))``, ``r`` and ``i`` sigmoids of
  block-diagonal products of ``u``; the state is multiplied by the gelu of another projection.
* ``attention``: queries and keys pass a causal convolution each, a key is also the value; a distance
  ``n`` takes ``r1_h ln(1 + r2_h n)`` off the score; window; one is added to the softmax's denominator; the heads'
  outputs times ``sigmoid(W_g h)``.
* ``delta``: the gated delta rule; q, k, v pass convolution and silu, q and k become unit vectors,
  ``S <- g S;  S <- S + k (beta (v - S^T k))^T;  o = S^T q``, a norm per head and ``silu(W_g h)``.

The feed-forward is ``W_down (g sigmoid(1.702 g) (u + 1))`` with ``g = min(W_gate h, L)``, ``u = clamp(W_up h, -L, L)``.

``dtype`` is the precision of matrix products and activations; the stream, norms, angles, scores, weights and
everything inside a recurrence stay in float32 (float64 when the whole run is).
"""

from __future__ import annotations

import math
from typing import Dict, List, Mapping, Optional

import torch


def _hi(x: torch.Tensor) -> torch.Tensor:
    return x if x.dtype == torch.float64 else x.float()


def _mm(x: torch.Tensor, w: torch.Tensor, dtype: torch.dtype) -> torch.Tensor:
    """``x W^T`` with operands in ``dtype``, summed in the high precision, rounded once to ``dtype``."""
    return (_hi(x.to(dtype)) @ _hi(w.to(dtype)).T).to(dtype)


# ------------------------------------------------------------------ mechanisms
def plain_rms(x: torch.Tensor, w: Optional[torch.Tensor], eps: float) -> torch.Tensor:
    x = _hi(x)
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if w is None else y * _hi(w)


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


def plain_softcap(s: torch.Tensor, cap: Optional[float]) -> torch.Tensor:
    return cap * torch.tanh(s / cap) if cap else s


def plain_weights_of(scores: torch.Tensor, visible: torch.Tensor, plus_one: bool = False) -> torch.Tensor:
    """``scores [H, T, T]`` to weights over the ``visible [T, T]`` keys; ``plus_one``: a one in the denominator."""
    s = scores.masked_fill(~visible[None], -math.inf)
    m = s.amax(-1, keepdim=True)
    if plus_one:
        m = m.clamp(min=0.0)
    e = torch.exp(s - m)
    den = e.sum(-1, keepdim=True)
    return e / (den + torch.exp(-m) if plus_one else den)


def plain_mix_heads(weights: torch.Tensor, talk: torch.Tensor) -> torch.Tensor:
    """``out[h] = sum_g talk[h, g] weights[g]`` for ``weights [H, T, T]``."""
    H = weights.shape[0]
    return (_hi(talk).to(weights.dtype) @ weights.reshape(H, -1)).reshape(weights.shape)


def plain_distance_bias(T: int, r1: torch.Tensor, r2: torch.Tensor) -> torch.Tensor:
    """``[H, query, key]``: ``r1_h ln(1 + r2_h n)`` for a key ``n`` tokens back."""
    i = torch.arange(T)
    n = (i[:, None] - i[None, :]).clamp(min=0).to(r1.dtype)
    return r1[:, None, None] * torch.log1p(r2[:, None, None] * n[None])


def plain_conv(u: torch.Tensor, taps: torch.Tensor, bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``y_t[c] = b[c] + sum_j taps[c, j] u_(t - K + 1 + j)[c]``, zeros before the start."""
    u, taps = _hi(u), _hi(taps)
    K = taps.shape[1]
    pad = torch.cat([u.new_zeros(K - 1, u.shape[1]), u])
    y = sum(pad[j : j + u.shape[0]] * taps[:, j].to(u.dtype) for j in range(K))
    return y if bias is None else y + _hi(bias)


def plain_heads_attend(a: torch.Tensor, v: torch.Tensor, dtype: torch.dtype) -> torch.Tensor:
    """``a [H, T, T]`` over values ``v [T, G, e]``: ``[T, H * e]``."""
    H, T, _ = a.shape
    G, e = v.shape[1], v.shape[2]
    out = torch.stack([a[h] @ _hi(v[:, h // (H // G)]) for h in range(H)], dim=1)
    return out.reshape(T, H * e)


def plain_scores(q: torch.Tensor, k: torch.Tensor, scale: float) -> torch.Tensor:
    H, G = q.shape[1], k.shape[1]
    return torch.stack([_hi(q[:, h]) @ _hi(k[:, h // (H // G)]).T for h in range(H)]) * scale


def plain_mixed_attention(x, w: Mapping[str, torch.Tensor], p: str, m: Mapping, eps: float, dtype: torch.dtype) -> torch.Tensor:
    """The parallel mixer's left half."""
    T, H, G, d, e = x.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = plain_rms(_mm(x, w[f"{p}.q"], dtype), w[f"{p}.q.norm"], eps).view(T, H, d)
    k = plain_rms(_mm(x, w[f"{p}.k"], dtype), w[f"{p}.k.norm"], eps).view(T, G, d)
    v = _mm(x, w[f"{p}.v"], dtype).view(T, G, e)
    q = plain_rotate(q, m["rot"]["base"], m["rot"]["dims"]).to(dtype)
    k = plain_rotate(k, m["rot"]["base"], m["rot"]["dims"]).to(dtype)
    s = plain_softcap(plain_scores(q, k, m["scale"]), m.get("softcap"))
    a = plain_weights_of(s, plain_window(T, (m.get("mask") or {}).get("size")))
    a = plain_mix_heads(a, w[f"{p}.talk"])
    return _mm(plain_heads_attend(a, v, dtype), w[f"{p}.o"], dtype)


def plain_lru(u: torch.Tensor, r: torch.Tensor, i: torch.Tensor, lam: torch.Tensor) -> torch.Tensor:
    """States ``[T, C]`` of ``S <- a S + sqrt(1 - a^2) i u``, ``a = exp(-8 r softplus(lam))``, from zero."""
    la = -8.0 * r * torch.nn.functional.softplus(lam)
    b = torch.sqrt(-torch.expm1(2 * la)) * i * u
    a = torch.exp(la)
    S, out = torch.zeros_like(u[0]), []
    for t in range(u.shape[0]):
        S = a[t] * S + b[t]
        out.append(S)
    return torch.stack(out)


def plain_block_linear(u: torch.Tensor, w: torch.Tensor, b: torch.Tensor, dtype: torch.dtype) -> torch.Tensor:
    """A block-diagonal product: ``w [blocks, out, in]``, ``b [blocks, out]``; not rounded."""
    B, n, _ = w.shape
    parts = _hi(u.to(dtype)).view(u.shape[0], B, n)
    return torch.cat([parts[:, j] @ _hi(w[j]).T + _hi(b[j]) for j in range(B)], dim=1)


def plain_gelu(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def plain_recurrent_block(x, w: Mapping[str, torch.Tensor], p: str, m: Mapping, dtype: torch.dtype) -> torch.Tensor:
    """The parallel mixer's right half."""
    y = plain_gelu(_hi(_mm(x, w[f"{p}.y"], dtype)) + _hi(w[f"{p}.y.b"]))
    u = _hi(_mm(x, w[f"{p}.x"], dtype)) + _hi(w[f"{p}.x.b"])
    u = _hi(plain_conv(u, w[f"{p}.conv"], w[f"{p}.conv.b"]).to(dtype))
    r = torch.sigmoid(plain_block_linear(u, w[f"{p}.ra"], w[f"{p}.ra.b"], dtype))
    i = torch.sigmoid(plain_block_linear(u, w[f"{p}.ri"], w[f"{p}.ri.b"], dtype))
    S = plain_lru(u, r, i, _hi(w[f"{p}.lam"]))
    return _mm((S * y).to(dtype), w[f"{p}.o"], dtype)


def plain_conv_attention(x, w: Mapping[str, torch.Tensor], p: str, m: Mapping, dtype: torch.dtype) -> torch.Tensor:
    T, H, G, d = x.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = plain_conv(_mm(x, w[f"{p}.q"], dtype), w[f"{p}.q.conv"]).to(dtype).view(T, H, d)
    k = plain_conv(_mm(x, w[f"{p}.k"], dtype), w[f"{p}.k.conv"]).to(dtype).view(T, G, d)
    s = plain_scores(q, k, m["scale"])
    s = s - plain_distance_bias(T, _hi(w[f"{p}.r1"]), _hi(w[f"{p}.r2"]))
    a = plain_weights_of(s, plain_window(T, (m.get("mask") or {}).get("size")), plus_one=True)
    o = plain_heads_attend(a, k, dtype) * torch.sigmoid(_hi(_mm(x, w[f"{p}.g"], dtype)))
    return _mm(o.to(dtype), w[f"{p}.o"], dtype)


def plain_delta_rule(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, g: torch.Tensor, beta: torch.Tensor) -> torch.Tensor:
    """One head: ``q, k [T, d]``, ``v [T, e]``, ``g, beta [T]`` -> ``o [T, e]``."""
    S, out = q.new_zeros(q.shape[1], v.shape[1]), []
    for t in range(q.shape[0]):
        S = g[t] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + k[t][:, None] * u[None, :]
        out.append(S.T @ q[t])
    return torch.stack(out)


def plain_silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def plain_unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def plain_delta_mixer(x, w: Mapping[str, torch.Tensor], p: str, m: Mapping, eps: float, dtype: torch.dtype) -> torch.Tensor:
    T, H, G, d, e = x.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    conv = lambda n: _hi(plain_silu(plain_conv(_mm(x, w[f"{p}.{n}"], dtype), w[f"{p}.{n}.conv"])).to(dtype))
    q = plain_unit(conv("q").view(T, G, d)) * d ** -0.5
    k = plain_unit(conv("k").view(T, G, d))
    v = conv("v").view(T, H, e)
    beta = torch.sigmoid(_hi(x.to(dtype)) @ _hi(w[f"{p}.b"]).T)
    a = _hi(x.to(dtype)) @ _hi(w[f"{p}.a"]).T + _hi(w[f"{p}.dt_bias"])
    g = torch.exp(-torch.exp(_hi(w[f"{p}.A_log"])) * torch.nn.functional.softplus(a))
    o = torch.stack([plain_delta_rule(q[:, h // (H // G)], k[:, h // (H // G)], v[:, h], g[:, h], beta[:, h])
                     for h in range(H)], dim=1)
    o = plain_rms(o, w[f"{p}.norm"], eps) * plain_silu(_hi(_mm(x, w[f"{p}.g"], dtype))).view(T, H, e)
    return _mm(o.reshape(T, H * e).to(dtype), w[f"{p}.o"], dtype)


def plain_feed_forward(x, w: Mapping[str, torch.Tensor], p: str, limit: float, dtype: torch.dtype) -> torch.Tensor:
    g = _hi(_mm(x, w[f"{p}.gate"], dtype)).clamp(max=limit)
    u = _hi(_mm(x, w[f"{p}.up"], dtype)).clamp(min=-limit, max=limit)
    return _mm((g * torch.sigmoid(1.702 * g) * (u + 1.0)).to(dtype), w[f"{p}.down"], dtype)


def plain_mixer(h, w, p: str, kind: str, m: Mapping, eps: float, dtype: torch.dtype) -> torch.Tensor:
    if kind == "parallel":
        left = _hi(plain_mixed_attention(h, w, f"{p}.left", m["left"], eps, dtype))
        right = _hi(plain_recurrent_block(h, w, f"{p}.right", m["right"], dtype))
        return m["left_scale"] * left + m["right_scale"] * right
    if kind == "attention":
        return _hi(plain_conv_attention(h, w, p, m, dtype))
    if kind == "delta":
        return _hi(plain_delta_mixer(h, w, p, m, eps, dtype))
    raise ValueError(kind)


# ----------------------------------------------------------------------- model
def plain_forward(weights: Mapping[str, torch.Tensor], config: Mapping, tokens: List[int],
                  dtype: torch.dtype = torch.float32, layers_out: Optional[list] = None) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one whole sequence.  ``layers_out``: a list that gets the stream after every layer."""
    if dtype == torch.float64:
        w = {k: v.double() if v.dtype.is_floating_point else v for k, v in weights.items()}
    else:
        w = {k: v.to(dtype) if v.dtype.is_floating_point else v for k, v in weights.items()}
    eps, mult = config["norm"]["eps"], config["residual_mult"]
    x = _hi(w["embed"][torch.tensor(tokens)]) * config["embedding"]["scale"]
    for i, layer in enumerate(config["layers"]):
        p = f"l{i}"
        h = plain_rms(x, 1.0 + _hi(w[f"{p}.norm1"]), eps).to(dtype)
        y = plain_mixer(h, w, f"{p}.mix", layer["type"], layer["mixer"], eps, dtype)
        x = x + mult * (y * _hi(w[f"{p}.ls1"]))
        if layer.get("mlp") is not None:
            h = plain_rms(x, 1.0 + _hi(w[f"{p}.norm2"]), eps).to(dtype)
            y = _hi(plain_feed_forward(h, w, f"{p}.mlp", layer["mlp"]["limit"], dtype))
            x = x + mult * (y * _hi(w[f"{p}.ls2"]))
        if layers_out is not None:
            layers_out.append(x)
    h = plain_rms(x, 1.0 + _hi(w["final.norm"]), eps).to(dtype)
    return _hi(h) @ _hi(w["embed"]).T


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
def plain_weights(config: Mapping, seed: int, stored: torch.dtype = torch.bfloat16) -> Dict[str, torch.Tensor]:
    """Random tensors of a configuration, by the names of the checkpoint, with the values that ``stored`` can hold
    (as float32)."""
    g = torch.Generator().manual_seed(seed)
    D, V = config["width"], config["vocab"]
    w: Dict[str, torch.Tensor] = {}

    def mat(name, rows, cols, std=None):
        w[name] = torch.randn(rows, cols, generator=g) * (std if std is not None else cols ** -0.5)

    def vec(name, *shape, mean=0.0, std=0.1):
        w[name] = mean + std * torch.randn(*shape, generator=g)

    mat("embed", V, D, 0.5)
    vec("final.norm", D)
    for i, layer in enumerate(config["layers"]):
        m, p = layer["mixer"], f"l{i}.mix"
        vec(f"l{i}.norm1", D)
        vec(f"l{i}.ls1", D, mean=1.0, std=0.2)
        if layer["type"] == "parallel":
            a, r = m["left"], m["right"]
            H, G, d, e, W, B = a["heads"], a["kv_heads"], a["dim"], a["vdim"], r["width"], r["blocks"]
            mat(f"{p}.left.q", H * d, D)
            mat(f"{p}.left.k", G * d, D)
            mat(f"{p}.left.v", G * e, D)
            vec(f"{p}.left.q.norm", H * d, mean=1.0, std=0.2)
            vec(f"{p}.left.k.norm", G * d, mean=1.0, std=0.2)
            w[f"{p}.left.talk"] = torch.eye(H) + 0.3 * torch.randn(H, H, generator=g)
            mat(f"{p}.left.o", D, H * e)
            for n in ("y", "x"):
                mat(f"{p}.right.{n}", W, D)
                vec(f"{p}.right.{n}.b", W, std=0.2)
            vec(f"{p}.right.conv", W, r["conv"], std=0.5)
            vec(f"{p}.right.conv.b", W, std=0.1)
            for n in ("ra", "ri"):
                vec(f"{p}.right.{n}", B, W // B, W // B, std=(W // B) ** -0.5)
                vec(f"{p}.right.{n}.b", B, W // B, std=0.5)
            vec(f"{p}.right.lam", W, mean=-4.0, std=1.5)
            mat(f"{p}.right.o", D, W)
        else:
            H, G, d, e, K = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
            if layer["type"] == "attention":
                mat(f"{p}.q", H * d, D)
                mat(f"{p}.k", G * d, D)
                vec(f"{p}.q.conv", H * d, K, std=0.6)
                vec(f"{p}.k.conv", G * d, K, std=0.6)
                w[f"{p}.r1"] = 0.2 + torch.rand(H, generator=g)
                w[f"{p}.r2"] = 0.05 + 0.5 * torch.rand(H, generator=g)
                mat(f"{p}.g", H * d, D)
                mat(f"{p}.o", D, H * d)
            else:
                mat(f"{p}.q", G * d, D)
                mat(f"{p}.k", G * d, D)
                mat(f"{p}.v", H * e, D)
                for n, c in (("q", G * d), ("k", G * d), ("v", H * e)):
                    vec(f"{p}.{n}.conv", c, K, std=0.6)
                mat(f"{p}.b", H, D)
                mat(f"{p}.a", H, D)
                vec(f"{p}.A_log", H, mean=-1.0, std=1.0)
                vec(f"{p}.dt_bias", H, mean=-2.0, std=1.0)
                vec(f"{p}.norm", e, mean=1.0, std=0.2)
                mat(f"{p}.g", H * e, D)
                mat(f"{p}.o", D, H * e)
        mlp = layer.get("mlp")
        if mlp is not None:
            vec(f"l{i}.norm2", D)
            vec(f"l{i}.ls2", D, mean=1.0, std=0.2)
            mat(f"l{i}.mlp.gate", mlp["ff"], D, 2 * D ** -0.5)
            mat(f"l{i}.mlp.up", mlp["ff"], D, 2 * D ** -0.5)
            mat(f"l{i}.mlp.down", D, mlp["ff"])
    return {k: v.to(stored).float() for k, v in w.items()}


# ---------------------------------------------------------------- configurations
def _parallel(heads, kv, dim, vdim, rot, window, softcap, width, blocks, conv, scales, base=900.0):
    left = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": dim ** -0.5}
    if rot:
        left["rot"] = {"base": base, "dims": rot}
    if window:
        left["mask"] = {"size": window}
    if softcap:
        left["softcap"] = softcap
    return {"left": left, "right": {"width": width, "blocks": blocks, "conv": conv}, "left_scale": scales[0],
            "right_scale": scales[1]}


def _attention(heads, kv, dim, window, conv):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "conv": conv}
    if window:
        m["mask"] = {"size": window}
    return m


def _delta(heads, kv, dim, vdim, conv):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}


def _model(width, vocab, layers, embed=3.0, mult=0.7, eps=1e-5):
    return {"architecture": "Ropelix", "width": width, "vocab": vocab, "embedding": {"scale": embed}, "residual_mult": mult,
            "norm": {"eps": eps}, "layers": [
                {"type": t, "mixer": m, "mlp": None if f is None else {"kind": "dense", "ff": f[0], "limit": f[1]}}
                for t, m, f in layers]}


# every mixer, one of each kind without a feed-forward
TRIO = _model(64, 96, [
    ("parallel", _parallel(4, 2, 16, 24, 8, 20, 8.0, 48, 3, 4, (0.8, 0.4)), (56, 1.5)),
    ("delta", _delta(4, 2, 16, 24, 3), (40, 0.9)),
    ("attention", _attention(4, 2, 16, 23, 2), (56, 1.5)),
    ("delta", _delta(3, 3, 32, 16, 2), None)])
# heads that are no power of two, a head size that is no multiple of 16 (or of 8), one key head a query head, values
# narrower than keys, every dimension rotated, no window, no cap, one block, one tap, widths that are no multiple of 8
ODD = _model(72, 50, [
    ("attention", _attention(3, 3, 20, None, 1), (44, 0.6)),
    ("parallel", _parallel(3, 3, 12, 6, 12, None, None, 36, 1, 1, (1.0, -0.5)), None),
    ("delta", _delta(6, 2, 10, 14, 1), (20, 2.0))], embed=1.0, mult=1.0, eps=1e-6)
# twenty heads (more than the matrix-core kernels mix or group) and twelve (one group), windows of one page
WIDE = _model(64, 80, [
    ("parallel", _parallel(20, 4, 8, 8, 4, 16, 3.0, 64, 4, 5, (0.5, 1.5)), (48, 1.0)),
    ("attention", _attention(20, 1, 8, 16, 4), (48, 1.0)),
    ("parallel", _parallel(12, 1, 16, 16, 6, 64, 12.0, 16, 2, 2, (1.3, 0.7)), (48, 1.0))])
ONLY_MIXED = _model(48, 64, [("parallel", _parallel(4, 2, 16, 16, 8, 32, None, 16, 2, 2, (1.0, 0.3)), None)], mult=1.0)
ONLY_CONV = _model(48, 64, [("attention", _attention(4, 1, 16, 32, 3), None)], mult=1.0)
ONLY_DELTA = _model(48, 64, [("delta", _delta(4, 2, 16, 16, 4), None)], mult=1.0)
