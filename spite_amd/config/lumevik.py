"""Typed configuration of the Lumevik design, read from the keys of its ``config.json``.

``architecture`` names the design; ``vocab``, ``width`` and ``norm.eps`` are the model's own; ``layers`` lists the
layers in order, each with its ``type`` (the kind of mixer), the mixer's sizes and constants under ``mixer`` and its
feed-forward under ``mlp`` (``null``: none).  Two kinds of mixer:

* ``attention``: grouped-query attention (``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``) with a learned bias by
  distance (``bias_max``: from where on all distances count alike), a sliding window whose request's first tokens stay
  in sight (``mask``: ``size``, ``keep_first``), a sink of score zero, and values blended with the first such layer's
  (``v_mix``);
* ``latent_attention``: attention over a cached latent without positions (``heads``, ``dim``, ``vdim``, ``kv_rank``,
  ``q_rank``, ``scale``).

Two kinds of feed-forward (``kind``), both gated with a bounded gate (``limit``): ``dense`` (``ff``) and ``moe``
(``router``: ``experts``, ``top``, ``groups.count``, ``groups.keep``; ``expert`` and ``shared``: ``ff``, ``limit``).
Every size and constant is read here; every problem found is reported in one ``ConfigError``.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional, Tuple, Union

from .llama4 import ConfigError

MIXER_TYPES = ("attention", "latent_attention")
MLP_KINDS = ("dense", "moe")


@dataclass(frozen=True)
class LumevikAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    bias_max: float
    window: Optional[int] = None          # mask.size; None: every earlier key
    keep_first: int = 0
    v_mix: bool = False


@dataclass(frozen=True)
class LumevikLatent:
    heads: int
    dim: int
    vdim: int
    kv_rank: int
    q_rank: int
    scale: float


@dataclass(frozen=True)
class LumevikDense:
    ff: int
    limit: float


@dataclass(frozen=True)
class LumevikMoe:
    experts: int
    top: int
    groups: Optional[Tuple[int, int]]     # (count, keep); None: one group
    expert: LumevikDense
    shared: Optional[LumevikDense]


@dataclass(frozen=True)
class LumevikLayer:
    type: str
    mixer: Union[LumevikAttention, LumevikLatent]
    mlp: Union[LumevikDense, LumevikMoe, None]


@dataclass(frozen=True)
class LumevikConfig:
    architecture: str
    vocab: int
    width: int
    norm_eps: float
    layers: Tuple[LumevikLayer, ...]
    torch_dtype: str = "bfloat16"
    eos_token_ids: Tuple[int, ...] = ()
    max_position: int = 1 << 20

    @staticmethod
    def from_dict(raw: Mapping[str, Any]) -> "LumevikConfig":
        problems = []

        def need(d, key, kind, where, least=None):
            if not isinstance(d, Mapping) or key not in d or d[key] is None:
                problems.append(f"{where}{key} is missing")
                return kind(1)
            try:
                v = kind(d[key])
            except (TypeError, ValueError):
                problems.append(f"{where}{key} = {d[key]!r} is no {kind.__name__}")
                return kind(1)
            if (least is None and not v > 0) or (least is not None and v < least):
                problems.append(f"{where}{key} = {v} must be " + ("positive" if least is None else f"at least {least}"))
            return v

        def gated(d, where):
            return LumevikDense(ff=need(d, "ff", int, where), limit=need(d, "limit", float, where))

        def attention(mx, w):
            mask = mx.get("mask")
            a = LumevikAttention(
                heads=need(mx, "heads", int, w), kv_heads=need(mx, "kv_heads", int, w), dim=need(mx, "dim", int, w),
                vdim=need(mx, "vdim", int, w), scale=need(mx, "scale", float, w), bias_max=need(mx, "bias_max", float, w),
                window=None if mask is None else need(mask, "size", int, w + "mask."),
                keep_first=0 if mask is None or mask.get("keep_first") is None else need(mask, "keep_first", int, w + "mask.", least=0),
                v_mix=bool(mx.get("v_mix", False)))
            if a.heads % a.kv_heads:
                problems.append(f"{w}heads = {a.heads} is no multiple of kv_heads = {a.kv_heads}")
            return a

        def moe(rm, w):
            router, shared, groups = rm.get("router") or {}, rm.get("shared"), (rm.get("router") or {}).get("groups")
            m = LumevikMoe(
                experts=need(router, "experts", int, w + "router."), top=need(router, "top", int, w + "router."),
                groups=None if groups is None else (need(groups, "count", int, w + "router.groups."), need(groups, "keep", int, w + "router.groups.")),
                expert=gated(rm.get("expert"), w + "expert."), shared=None if shared is None else gated(shared, w + "shared."))
            count, keep = m.groups or (1, 1)
            if m.experts % count:
                problems.append(f"{w}router.groups.count = {count} does not divide {m.experts} experts")
            elif keep > count:
                problems.append(f"{w}router.groups.keep = {keep} of {count} groups")
            elif m.top > keep * (m.experts // count):
                problems.append(f"{w}router.top = {m.top} of {keep * (m.experts // count)} experts that can be chosen")
            return m

        layers = []
        raw_layers = raw.get("layers")
        if not isinstance(raw_layers, (list, tuple)) or not raw_layers:
            problems.append("layers is missing or empty")
            raw_layers = []
        for i, L in enumerate(raw_layers):
            w = f"layers[{i}]."
            kind = L.get("type") if isinstance(L, Mapping) else None
            if kind not in MIXER_TYPES:
                problems.append(f"{w}type = {kind!r} (known: {', '.join(MIXER_TYPES)})")
                continue
            mx, wm = L.get("mixer") or {}, w + "mixer."
            if kind == "attention":
                mixer = attention(mx, wm)
            else:
                mixer = LumevikLatent(heads=need(mx, "heads", int, wm), dim=need(mx, "dim", int, wm), vdim=need(mx, "vdim", int, wm),
                                      kv_rank=need(mx, "kv_rank", int, wm), q_rank=need(mx, "q_rank", int, wm),
                                      scale=need(mx, "scale", float, wm))
            mlp, rm = None, L.get("mlp")
            if rm is not None:
                wl = w + "mlp."
                if rm.get("kind") not in MLP_KINDS:
                    problems.append(f"{wl}kind = {rm.get('kind')!r} (known: {', '.join(MLP_KINDS)})")
                else:
                    mlp = gated(rm, wl) if rm["kind"] == "dense" else moe(rm, wl)
            layers.append(LumevikLayer(kind, mixer, mlp))
        blended = {(l.mixer.kv_heads, l.mixer.vdim) for l in layers if l.type == "attention" and l.mixer.v_mix}
        if len(blended) > 1:
            problems.append(f"layers with v_mix differ in (kv_heads, vdim): {sorted(blended)}; their values are blended one by one")
        cfg = LumevikConfig(
            architecture=str(raw.get("architecture", "Lumevik")),
            vocab=need(raw, "vocab", int, ""), width=need(raw, "width", int, ""),
            norm_eps=need(raw.get("norm") or {}, "eps", float, "norm."), layers=tuple(layers),
            torch_dtype=str(raw.get("torch_dtype", "bfloat16")),
            eos_token_ids=tuple(int(t) for t in raw.get("eos_token_ids", ()) or ()),
            max_position=int(raw.get("max_position", 1 << 20)))
        if problems:
            raise ConfigError("config.json does not describe a Lumevik model: " + "; ".join(problems))
        return cfg
