"""The Ropelix decoder as a layout of parts.

A Ropelix ``config.json`` is nested: ``width``, ``vocab``, ``embedding.scale``, ``residual_mult``, ``norm.eps`` and a list
``layers`` whose entries name their mixer (``type``), its sizes (``mixer``) and their feed-forward (``mlp``: ``{"kind":
"dense", "ff": n, "limit": x}`` or null).  Every layer is pre-norm with norm weights stored around zero; each
sublayer's output is multiplied per channel by ``l<i>.ls1`` / ``ls2`` and by ``residual_mult`` before it is added.  The head
is the embedding table (without its scale).

* ``parallel``: two mixers on the same input, ``left_scale`` times the one plus ``right_scale`` times the other.  ``left``
  is softmax attention with norms over the whole q and k projections, a rotation of the first ``rot.dims`` dimensions
  (pairs ``i, i + dims/2``), soft-capped scores, a sliding window (``mask.size``), and the heads' weights mixed by ``talk``
  after the softmax; ``right`` is a recurrent block with a real-gated linear recurrent unit (``width``, ``blocks``,
  ``conv`` taps).
* ``attention``: queries and keys behind short convolutions (``conv`` taps), a key is also the value (``vdim`` equals
  ``dim``), a logarithmic distance bias (``r1``, ``r2``), a window, one more in the softmax's denominator, an output gate.
* ``delta``: the gated delta rule behind short convolutions.

Tensors are named ``embed``, ``l<i>.{norm1,norm2,ls1,ls2}``, ``l<i>.mix.*`` (``l<i>.mix.left.*`` and ``l<i>.mix.right.*`` in a
parallel layer), ``l<i>.mlp.{gate,up,down}``, ``final.norm``.
"""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Mapping, Optional, Tuple, Union

from .buderax import _get
from .layout import LayerSpec, ModelLayout, PartSpec, RunEntry
from .model_args import ConfigError
from .registry import register_architecture

SWISH_ALPHA = 1.702  # the feed-forward's activation is g * sigmoid(1.702 g) * (u + 1)
DECAY_SCALE = 8.0  # log a = -8 r softplus(lam)
UNIT_EPS = 1e-6  # inside the root of the unit vectors' norm


@dataclass(frozen=True)
class MixedAttentionArgs:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: Optional[float]
    window: Optional[int]
    rot_dims: int
    rot_base: float


@dataclass(frozen=True)
class RecurrentArgs:
    width: int
    blocks: int
    conv: int


@dataclass(frozen=True)
class ParallelArgs:
    left: MixedAttentionArgs
    right: RecurrentArgs
    left_scale: float
    right_scale: float


@dataclass(frozen=True)
class ConvAttentionArgs:
    heads: int
    kv_heads: int
    dim: int
    scale: float
    window: Optional[int]
    conv: int


@dataclass(frozen=True)
class DeltaArgs:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int


@dataclass(frozen=True)
class DenseArgs:
    ff: int
    limit: float


@dataclass(frozen=True)
class RopelixLayer:
    type: str
    mixer: Union[ParallelArgs, ConvAttentionArgs, DeltaArgs]
    mlp: Optional[DenseArgs]


@dataclass(frozen=True)
class RopelixArgs:
    architecture: str
    width: int
    vocab: int
    embedding_scale: float
    residual_mult: float
    norm_eps: float
    layers: Tuple[RopelixLayer, ...]
    extra: Mapping[str, Any] = field(default_factory=dict, compare=False)

    @property
    def vocab_size(self) -> int:
        return self.vocab


def _check(where: str, args: Any, *positive: str) -> None:
    for name in positive:
        v = getattr(args, name)
        if v is not None and not v > 0:
            raise ConfigError(f"config.json: {where}.{name}={v} must be positive")
    if hasattr(args, "kv_heads") and args.heads % args.kv_heads:
        raise ConfigError(f"config.json: {where}: heads={args.heads} is not a multiple of kv_heads={args.kv_heads}")


def _parallel(m: Mapping[str, Any], where: str) -> ParallelArgs:
    l, r = _get(m, "left"), _get(m, "right")
    left = MixedAttentionArgs(
        _get(l, "heads", int), _get(l, "kv_heads", int), _get(l, "dim", int), _get(l, "vdim", int), _get(l, "scale", float),
        _get(l, "softcap", float, None), _get(l, "mask.size", int, None), _get(l, "rot.dims", int, 0),
        _get(l, "rot.base", float, 10000.0))
    _check(f"{where}.left", left, "heads", "kv_heads", "dim", "vdim", "scale", "softcap", "window", "rot_base")
    if left.rot_dims % 2 or not 0 <= left.rot_dims <= left.dim:
        raise ConfigError(f"config.json: {where}.left: rot.dims={left.rot_dims} must be even and at most dim={left.dim}")
    right = RecurrentArgs(_get(r, "width", int), _get(r, "blocks", int), _get(r, "conv", int))
    _check(f"{where}.right", right, "width", "blocks", "conv")
    if right.width % right.blocks:
        raise ConfigError(f"config.json: {where}.right: width={right.width} is not a multiple of blocks={right.blocks}")
    return ParallelArgs(left, right, _get(m, "left_scale", float, 1.0), _get(m, "right_scale", float, 1.0))


def _attention(m: Mapping[str, Any], where: str) -> ConvAttentionArgs:
    a = ConvAttentionArgs(_get(m, "heads", int), _get(m, "kv_heads", int), _get(m, "dim", int), _get(m, "scale", float),
                          _get(m, "mask.size", int, None), _get(m, "conv", int))
    _check(where, a, "heads", "kv_heads", "dim", "scale", "window", "conv")
    vdim = _get(m, "vdim", int, a.dim)
    if vdim != a.dim:
        raise ConfigError(f"config.json: {where}: the values are the keys, so vdim={vdim} must equal dim={a.dim}")
    return a


def _delta(m: Mapping[str, Any], where: str) -> DeltaArgs:
    a = DeltaArgs(_get(m, "heads", int), _get(m, "kv_heads", int), _get(m, "dim", int), _get(m, "vdim", int), _get(m, "conv", int))
    _check(where, a, "heads", "kv_heads", "dim", "vdim", "conv")
    return a


_MIXERS = {"parallel": _parallel, "attention": _attention, "delta": _delta}


class RopelixArchitecture:
    name = "Ropelix"

    def parse(self, config: Mapping[str, Any]) -> RopelixArgs:
        layers = []
        for i, l in enumerate(_get(config, "layers")):
            kind = _get(l, "type", str)
            if kind not in _MIXERS:
                raise ConfigError(f"config.json: layers[{i}].type {kind!r} is not supported (supported: {sorted(_MIXERS)})")
            mixer = _MIXERS[kind](_get(l, "mixer"), f"layers[{i}].mixer")
            mlp, ff = l.get("mlp"), None
            if mlp is not None:
                if mlp.get("kind", "dense") != "dense":
                    raise ConfigError(f"config.json: layers[{i}].mlp.kind {mlp.get('kind')!r} is not supported (supported: 'dense')")
                ff = DenseArgs(_get(mlp, "ff", int), _get(mlp, "limit", float))
                _check(f"layers[{i}].mlp", ff, "ff", "limit")
            layers.append(RopelixLayer(kind, mixer, ff))
        return RopelixArgs(
            architecture=self.name, width=_get(config, "width", int), vocab=_get(config, "vocab", int),
            embedding_scale=_get(config, "embedding.scale", float, 1.0), residual_mult=_get(config, "residual_mult", float, 1.0),
            norm_eps=_get(config, "norm.eps", float), layers=tuple(layers),
            extra={k: config[k] for k in ("bos_token_id", "eos_token_id") if k in config},
        )

    def to_hf_config(self, args: RopelixArgs) -> dict:
        mask = lambda a: {} if a.window is None else {"mask": {"size": a.window}}

        def mixer(l: RopelixLayer) -> dict:
            m = l.mixer
            if l.type == "parallel":
                a, r = m.left, m.right
                left = {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim, "scale": a.scale, **mask(a)}
                if a.softcap is not None:
                    left["softcap"] = a.softcap
                if a.rot_dims:
                    left["rot"] = {"base": a.rot_base, "dims": a.rot_dims}
                return {"left": left, "right": {"width": r.width, "blocks": r.blocks, "conv": r.conv},
                        "left_scale": m.left_scale, "right_scale": m.right_scale}
            if l.type == "attention":
                return {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.dim, "scale": m.scale, "conv": m.conv,
                        **mask(m)}
            return {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "conv": m.conv}

        out = {"architecture": self.name, "width": args.width, "vocab": args.vocab, "embedding": {"scale": args.embedding_scale},
               "residual_mult": args.residual_mult, "norm": {"eps": args.norm_eps},
               "layers": [{"type": l.type, "mixer": mixer(l),
                           "mlp": None if l.mlp is None else {"kind": "dense", "ff": l.mlp.ff, "limit": l.mlp.limit}}
                          for l in args.layers]}
        out.update(args.extra)
        return out

    def layout(self, args: RopelixArgs) -> ModelLayout:
        bare = {"weight": ""}  # a part's one tensor is named by the prefix alone
        D, eps = args.width, args.norm_eps

        def norm(prefix: str) -> PartSpec:
            return PartSpec("rmsnorm", prefix, dict(dim=D, eps=eps, unit_offset=True, names=bare))

        def mixer(l: RopelixLayer, p: str) -> PartSpec:
            m = l.mixer
            if l.type == "parallel":
                a, r = m.left, m.right
                rope = (PartSpec("rope", options=dict(head_dim=a.dim, rotary_dim=a.rot_dims, theta=a.rot_base, pairing="half"))
                        if a.rot_dims else PartSpec("none"))
                left = PartSpec("mixed_attention", f"{p}.left", dict(
                    dim=D, n_heads=a.heads, n_kv_heads=a.kv_heads, head_dim=a.dim, v_head_dim=a.vdim, scale=a.scale,
                    softcap=a.softcap, window=a.window, eps=eps, position=rope,
                    names={"q_proj.weight": "q", "k_proj.weight": "k", "v_proj.weight": "v", "o_proj.weight": "o",
                           "q_norm.weight": "q.norm", "k_norm.weight": "k.norm", "head_mix": "talk"}))
                right = PartSpec("gated_linear_recurrence", f"{p}.right", dict(
                    dim=D, width=r.width, blocks=r.blocks, taps=r.conv, decay_scale=DECAY_SCALE,
                    names={"y_proj.weight": "y", "y_proj.bias": "y.b", "x_proj.weight": "x", "x_proj.bias": "x.b",
                           "conv.weight": "conv", "conv.bias": "conv.b", "r_gate.weight": "ra", "r_gate.bias": "ra.b",
                           "i_gate.weight": "ri", "i_gate.bias": "ri.b", "decay": "lam", "o_proj.weight": "o"}))
                return PartSpec("parallel_mixers", p, dict(dim=D, left=left, right=right, left_scale=m.left_scale,
                                                           right_scale=m.right_scale))
            if l.type == "attention":
                return PartSpec("attention", p, dict(
                    dim=D, n_heads=m.heads, n_kv_heads=m.kv_heads, head_dim=m.dim, scale=m.scale, window=m.window,
                    position=PartSpec("none"), value_from_key=True, output_gate=True, exact_weights=True, sink="one",
                    conv_taps=m.conv, distance_bias=True,
                    names={"q_proj.weight": "q", "k_proj.weight": "k", "o_proj.weight": "o", "gate_proj.weight": "g",
                           "q_conv.weight": "q.conv", "k_conv.weight": "k.conv", "distance.r1": "r1", "distance.r2": "r2"}))
            return PartSpec("gated_delta_rule", p, dict(
                dim=D, n_heads=m.heads, n_kv_heads=m.kv_heads, head_dim=m.dim, v_head_dim=m.vdim, taps=m.conv, eps=eps,
                unit_eps=UNIT_EPS,
                names={"q_proj.weight": "q", "k_proj.weight": "k", "v_proj.weight": "v", "q_conv.weight": "q.conv",
                       "k_conv.weight": "k.conv", "v_conv.weight": "v.conv", "gate_proj.weight": "g", "beta_proj.weight": "b",
                       "decay_proj.weight": "a", "out_norm.weight": "norm", "o_proj.weight": "o"}))

        layers, order = [], []
        for i, l in enumerate(args.layers):
            ffn = None
            if l.mlp is not None:
                ffn = PartSpec("swiglu", f"l{i}.mlp", dict(
                    dim=D, hidden_dim=l.mlp.ff, activation="limited", limit=l.mlp.limit, alpha=SWISH_ALPHA,
                    names={"gate_proj.weight": "gate", "up_proj.weight": "up", "down_proj.weight": "down"}))
            layers.append(LayerSpec(
                mixer=mixer(l, f"l{i}.mix"), ffn=ffn, mixer_norm=norm(f"l{i}.norm1"),
                ffn_norm=norm(f"l{i}.norm2") if ffn is not None else None, arrangement="pre_norm_scaled",
                arrangement_spec=PartSpec("pre_norm_scaled", f"l{i}", dict(dim=D, mult=args.residual_mult))))
            order.append(RunEntry(i))
        return ModelLayout(
            dim=D, vocab_size=args.vocab,
            embed=PartSpec("embedding", "embed", dict(vocab_size=args.vocab, dim=D, scale=args.embedding_scale, names=bare)),
            layers=tuple(layers), order=tuple(order), final_norm=norm("final.norm"),
            head=PartSpec("lm_head", "head", dict(vocab_size=args.vocab, dim=D, tied_to="embed", names=bare)),
        )


ROPELIX = register_architecture(RopelixArchitecture())
