"""The Poselorn decoder as a layout of parts.

A Poselorn ``config.json`` is nested: ``width``, ``vocab``, ``embedding.scale``, ``residual_mult``, ``norm.eps``, a list
``layers`` whose entries name their mixer (``type``), its sizes (``mixer``) and their feed-forward (``mlp``, or null), and
optionally ``loop``, a stretch of layers (``start`` to before ``stop``) that is repeated, ``times`` passes over one set of
weights, each pass with storage of its own; every pass but the first begins by adding the embedding's output.  In a layer both sublayers read the same stream through norms of
their own, and their outputs, scaled per channel (``l<i>.ls1`` / ``ls2``) and by ``residual_mult``, are added at once.

* ``channel_delta``: the gated delta rule behind short convolutions (``conv`` taps) with a decay per key channel; the decays and
  the output gate are projections through narrow middles, whose widths are no keys of the configuration: they are the
  shapes of ``l<i>.mix.a1`` and ``l<i>.mix.g1`` (``parse`` takes the tensors' shapes), or the optional keys ``decay_rank`` and
  ``gate_rank`` where there are no tensors yet.
* ``parallel``: windowed attention (``left``: biases, norms per head, partial rotation, ``mask.size``) and linear attention with
  a constant decay per head (``right``) on one input; each output is normed, and half their sum is the mixer's.

The feed-forward is ``{"kind": "dense", "ff": n}`` (square of ReLU, biases) or ``{"kind": "moe", "expert": {"ff": n}, "router":
{"experts", "top", "identity", "groups": {"count", "keep"}}}``: softmax scores over experts and identity experts together, a
correction in the choice, groups ranked by their best, weights not renormalized.  The head is a matrix of its own.  Tensors
are named ``embed``, ``l<i>.{norm1,norm2,ls1,ls2}``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``, ``head``.
"""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Callable, Mapping, Optional, Tuple, Union

from .buderax import LoopArgs, _get
from .layout import LayerSpec, ModelLayout, PartSpec, RunEntry
from .model_args import ConfigError
from .registry import register_architecture

DEFAULT_RANK = 16
UNIT_EPS = 1e-6  # inside the root of the unit vectors' norm
SIDE_WEIGHT = 0.5  # of each of the two normed outputs of a parallel mixer


@dataclass(frozen=True)
class ChannelDeltaArgs:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    decay_rank: int
    gate_rank: int


@dataclass(frozen=True)
class WindowArgs:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int]
    rot_dims: int
    rot_base: float


@dataclass(frozen=True)
class LightningArgs:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]


@dataclass(frozen=True)
class SidesArgs:
    left: WindowArgs
    right: LightningArgs


@dataclass(frozen=True)
class DenseArgs:
    ff: int


@dataclass(frozen=True)
class RoutedArgs:
    experts: int
    identity: int
    top: int
    ff: int
    groups: int
    keep: int


@dataclass(frozen=True)
class PoselornLayer:
    type: str
    mixer: Union[ChannelDeltaArgs, SidesArgs]
    mlp: Union[DenseArgs, RoutedArgs, None]


@dataclass(frozen=True)
class PoselornArgs:
    architecture: str
    width: int
    vocab: int
    embedding_scale: float
    residual_mult: float
    norm_eps: float
    layers: Tuple[PoselornLayer, ...]
    loop: Optional[LoopArgs]
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


def _sides(m: Mapping[str, Any], where: str) -> SidesArgs:
    l, r = _get(m, "left"), _get(m, "right")
    left = WindowArgs(_get(l, "heads", int), _get(l, "kv_heads", int), _get(l, "dim", int), _get(l, "vdim", int),
                      _get(l, "scale", float), _get(l, "mask.size", int, None), _get(l, "rot.dims", int, 0),
                      _get(l, "rot.base", float, 10000.0))
    _check(f"{where}.left", left, "heads", "kv_heads", "dim", "vdim", "scale", "window", "rot_base")
    if left.rot_dims % 2 or not 0 <= left.rot_dims <= left.dim:
        raise ConfigError(f"config.json: {where}.left: rot.dims={left.rot_dims} must be even and at most dim={left.dim}")
    right = LightningArgs(_get(r, "heads", int), _get(r, "dim", int), _get(r, "vdim", int), tuple(float(x) for x in _get(r, "decay")))
    _check(f"{where}.right", right, "heads", "dim", "vdim")
    if len(right.decay) != right.heads or not all(0 <= x <= 1 for x in right.decay):
        raise ConfigError(f"config.json: {where}.right.decay must hold a number between 0 and 1 for each of the {right.heads} heads")
    return SidesArgs(left, right)


def _mlp(mlp: Mapping[str, Any], where: str) -> Union[DenseArgs, RoutedArgs]:
    kind = _get(mlp, "kind", str)
    if kind == "dense":
        d = DenseArgs(_get(mlp, "ff", int))
        _check(where, d, "ff")
        return d
    if kind != "moe":
        raise ConfigError(f"config.json: {where}.kind {kind!r} is not supported (supported: 'dense', 'moe')")
    groups = _get(mlp, "router.groups.count", int, 1)
    a = RoutedArgs(_get(mlp, "router.experts", int), _get(mlp, "router.identity", int, 0), _get(mlp, "router.top", int),
                   _get(mlp, "expert.ff", int), groups, _get(mlp, "router.groups.keep", int, groups))
    _check(where, a, "experts", "top", "ff", "groups", "keep")
    scored = a.experts + a.identity
    if a.identity < 0 or scored % a.groups or a.keep > a.groups or a.top > a.keep * (scored // a.groups):
        raise ConfigError(f"config.json: {where}: {a.groups} groups of which {a.keep} stay do not fit {scored} experts and top={a.top}")
    return a


class PoselornArchitecture:
    name = "Poselorn"

    def parse(self, config: Mapping[str, Any], shape_of: Optional[Callable[[str], Optional[Tuple[int, ...]]]] = None
              ) -> PoselornArgs:
        """``shape_of(name)``: the shape of a tensor of the checkpoint (None if it has none of that name); sizes that only
        the tensors give are read from it."""
        layers = []
        for i, l in enumerate(_get(config, "layers")):
            kind, m, where = _get(l, "type", str), _get(l, "mixer"), f"layers[{i}].mixer"
            if kind == "parallel":
                a: Union[ChannelDeltaArgs, SidesArgs] = _sides(m, where)
            elif kind == "channel_delta":
                ranks = []
                for key, tensor in (("decay_rank", "a1"), ("gate_rank", "g1")):
                    shape = shape_of(f"l{i}.mix.{tensor}") if shape_of is not None else None
                    ranks.append(int(shape[0]) if shape is not None else _get(m, key, int, DEFAULT_RANK))
                a = ChannelDeltaArgs(_get(m, "heads", int), _get(m, "kv_heads", int), _get(m, "dim", int), _get(m, "vdim", int),
                                     _get(m, "conv", int), *ranks)
                _check(where, a, "heads", "kv_heads", "dim", "vdim", "conv", "decay_rank", "gate_rank")
            else:
                raise ConfigError(f"config.json: layers[{i}].type {kind!r} is not supported"
                                  " (supported: 'channel_delta', 'parallel')")
            mlp = l.get("mlp")
            layers.append(PoselornLayer(kind, a, None if mlp is None else _mlp(mlp, f"layers[{i}].mlp")))
        loop = None
        if config.get("loop") is not None:
            loop = LoopArgs(_get(config, "loop.start", int), _get(config, "loop.stop", int), _get(config, "loop.times", int))
            if not 0 <= loop.start < loop.stop <= len(layers) or loop.times < 1:
                raise ConfigError(f"config.json: loop start={loop.start} stop={loop.stop} times={loop.times} does not fit"
                                  f" {len(layers)} layers")
        return PoselornArgs(
            architecture=self.name, width=_get(config, "width", int), vocab=_get(config, "vocab", int),
            embedding_scale=_get(config, "embedding.scale", float, 1.0), residual_mult=_get(config, "residual_mult", float, 1.0),
            norm_eps=_get(config, "norm.eps", float), layers=tuple(layers), loop=loop,
            extra={k: config[k] for k in ("bos_token_id", "eos_token_id") if k in config},
        )

    def to_hf_config(self, args: PoselornArgs) -> dict:
        def mixer(m: Union[ChannelDeltaArgs, SidesArgs]) -> dict:
            if isinstance(m, ChannelDeltaArgs):
                return {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "conv": m.conv,
                        "decay_rank": m.decay_rank, "gate_rank": m.gate_rank}
            a, r = m.left, m.right
            left = {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim, "scale": a.scale}
            if a.window is not None:
                left["mask"] = {"size": a.window}
            if a.rot_dims:
                left["rot"] = {"base": a.rot_base, "dims": a.rot_dims}
            return {"left": left, "right": {"heads": r.heads, "dim": r.dim, "vdim": r.vdim, "decay": list(r.decay)}}

        def mlp(f: Union[DenseArgs, RoutedArgs, None]) -> Optional[dict]:
            if f is None:
                return None
            if isinstance(f, DenseArgs):
                return {"kind": "dense", "ff": f.ff}
            return {"kind": "moe", "expert": {"ff": f.ff}, "router": {
                "experts": f.experts, "identity": f.identity, "top": f.top, "groups": {"count": f.groups, "keep": f.keep}}}

        out = {"architecture": self.name, "width": args.width, "vocab": args.vocab, "embedding": {"scale": args.embedding_scale},
               "residual_mult": args.residual_mult, "norm": {"eps": args.norm_eps},
               "layers": [{"type": l.type, "mixer": mixer(l.mixer), "mlp": mlp(l.mlp)} for l in args.layers]}
        if args.loop is not None:
            out["loop"] = {"start": args.loop.start, "stop": args.loop.stop, "times": args.loop.times}
        out.update(args.extra)
        return out

    def layout(self, args: PoselornArgs) -> ModelLayout:
        bare = {"weight": ""}  # a part's one tensor is named by the prefix alone
        D, eps = args.width, args.norm_eps

        def norm(prefix: str) -> PartSpec:
            return PartSpec("rmsnorm", prefix, dict(dim=D, eps=eps, names=bare))

        def mixer(m: Union[ChannelDeltaArgs, SidesArgs], p: str) -> PartSpec:
            if isinstance(m, ChannelDeltaArgs):
                return PartSpec("channel_delta_rule", p, dict(
                    dim=D, n_heads=m.heads, n_kv_heads=m.kv_heads, head_dim=m.dim, v_head_dim=m.vdim, taps=m.conv, eps=eps,
                    unit_eps=UNIT_EPS, decay_rank=m.decay_rank, gate_rank=m.gate_rank,
                    names={"q_proj.weight": "q", "k_proj.weight": "k", "v_proj.weight": "v", "q_conv.weight": "q.conv",
                           "k_conv.weight": "k.conv", "v_conv.weight": "v.conv", "beta_proj.weight": "b", "decay_down.weight": "a1",
                           "decay_up.weight": "a2", "gate_down.weight": "g1", "gate_up.weight": "g2", "out_norm.weight": "norm",
                           "o_proj.weight": "o"}))
            a, r = m.left, m.right
            rope = (PartSpec("rope", options=dict(head_dim=a.dim, rotary_dim=a.rot_dims, theta=a.rot_base, pairing="half"))
                    if a.rot_dims else PartSpec("none"))
            left = PartSpec("attention", f"{p}.left", dict(
                dim=D, n_heads=a.heads, n_kv_heads=a.kv_heads, head_dim=a.dim, v_head_dim=a.vdim, scale=a.scale, window=a.window,
                position=rope, bias=True, qk_norm=True, qk_norm_eps=eps, exact_weights=True,
                names={"q_proj.weight": "q", "k_proj.weight": "k", "v_proj.weight": "v", "o_proj.weight": "o", "q_proj.bias": "q.b",
                       "k_proj.bias": "k.b", "v_proj.bias": "v.b", "q_norm.weight": "q.norm", "k_norm.weight": "k.norm"}))
            right = PartSpec("lightning_attention", f"{p}.right", dict(
                dim=D, n_heads=r.heads, head_dim=r.dim, v_head_dim=r.vdim, decay=r.decay, eps=eps,
                names={"q_proj.weight": "q", "k_proj.weight": "k", "v_proj.weight": "v", "gate_proj.weight": "g",
                       "out_norm.weight": "norm", "o_proj.weight": "o"}))
            return PartSpec("parallel_mixers", p, dict(
                dim=D, left=left, right=right, left_scale=SIDE_WEIGHT, right_scale=SIDE_WEIGHT, out_norms=True, eps=eps,
                names={"left_norm.weight": "left.out", "right_norm.weight": "right.out"}))

        layers = []
        for i, l in enumerate(args.layers):
            f, p, ffn = l.mlp, f"l{i}.mlp", None
            if isinstance(f, DenseArgs):
                ffn = PartSpec("mlp", p, dict(dim=D, hidden_dim=f.ff, activation="relu2", bias=True, names={
                    "up_proj.weight": "up", "up_proj.bias": "up.b", "down_proj.weight": "down", "down_proj.bias": "down.b"}))
            elif f is not None:
                ffn = PartSpec("moe", p, dict(
                    dim=D, hidden_dim=f.ff, n_experts=f.experts, identity=f.identity, top=f.top, router_bias=False,
                    scoring="softmax_all", correction=True, n_groups=f.groups, keep_groups=f.keep, group_rank="max",
                    renormalize=False, names={"router.weight": "router", "expert": "e{}", "gate_proj.weight": "gate",
                                              "up_proj.weight": "up", "down_proj.weight": "down"}))
            layers.append(LayerSpec(
                mixer=mixer(l.mixer, f"l{i}.mix"), ffn=ffn, mixer_norm=norm(f"l{i}.norm1"),
                ffn_norm=norm(f"l{i}.norm2") if ffn is not None else None, arrangement="parallel_scaled",
                arrangement_spec=PartSpec("parallel_scaled", f"l{i}", dict(dim=D, mult=args.residual_mult))))
        n, lp = len(layers), args.loop
        injections: Tuple[PartSpec, ...] = ()
        if lp is None or lp.times == 1:
            order = [RunEntry(i) for i in range(n)]
        else:
            injections = (PartSpec("loop_input", "loop", dict(dim=D, times=lp.times, table=False)),)
            order = [RunEntry(i) for i in range(lp.start)]
            for t in range(lp.times):
                order += [RunEntry(i, inject=(0, t) if t and i == lp.start else None) for i in range(lp.start, lp.stop)]
            order += [RunEntry(i) for i in range(lp.stop, n)]
        return ModelLayout(
            dim=D, vocab_size=args.vocab,
            embed=PartSpec("embedding", "embed", dict(vocab_size=args.vocab, dim=D, scale=args.embedding_scale, names=bare)),
            layers=tuple(layers), order=tuple(order), final_norm=norm("final.norm"),
            head=PartSpec("lm_head", "head", dict(vocab_size=args.vocab, dim=D, tied_to=None, names=bare)),
            injections=injections,
        )


POSELORN = register_architecture(PoselornArchitecture())
