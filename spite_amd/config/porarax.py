"""Typed configuration of the Porarax design, read from the keys of its ``config.json``.

``architecture`` names the design; ``vocab``, ``width`` and ``norm.eps`` are the model's own; ``layers`` lists the
layers in order, each with its ``type`` (the kind of mixer), the mixer's sizes and constants under ``mixer`` and its
feed-forward under ``mlp`` (``null``: none).  Three kinds of mixer:

* ``latent_attention``: attention over a cached latent without positions (``heads``, ``dim``, ``vdim``, ``kv_rank``,
  ``q_rank``, ``scale``), under a sliding window (``mask.size``; no mask: every earlier key), over the layer's own latent
  or an earlier layer's (``kv_from``);
* ``attention``: grouped-query attention (``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``) with a rotation of a head's
  leading part (``rot``: ``base``, ``dims``; no ``rot``: none), normed queries and keys and a gate on every element;
* ``delta``: the gated delta rule (``heads``, ``kv_heads``, ``dim``, ``vdim``, ``conv``: the convolution's taps).

The feed-forward (``kind`` ``moe``): ``router.experts``, ``router.top``, ``expert.ff``, ``expert.limit``.
Every size and constant is read here; every problem found is reported in one ``ConfigError``.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional, Tuple, Union

from .llama4 import ConfigError

MIXER_TYPES = ("latent_attention", "attention", "delta")


@dataclass(frozen=True)
class PoraraxLatent:
    heads: int
    dim: int
    vdim: int
    kv_rank: int
    q_rank: int
    scale: float
    window: Optional[int] = None          # mask.size; None: every earlier key
    kv_from: Optional[int] = None         # the layer whose latent this one reads; None: its own


@dataclass(frozen=True)
class PoraraxAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_base: Optional[float] = None
    rot_dims: int = 0


@dataclass(frozen=True)
class PoraraxDelta:
    heads: int
    kv_heads: int                         # heads of q and k
    dim: int
    vdim: int
    conv: int


@dataclass(frozen=True)
class PoraraxMoe:
    experts: int
    top: int
    ff: int
    limit: float


@dataclass(frozen=True)
class PoraraxLayer:
    type: str
    mixer: Union[PoraraxLatent, PoraraxAttention, PoraraxDelta]
    mlp: Optional[PoraraxMoe]


@dataclass(frozen=True)
class PoraraxConfig:
    architecture: str
    vocab: int
    width: int
    norm_eps: float
    layers: Tuple[PoraraxLayer, ...]
    torch_dtype: str = "bfloat16"
    eos_token_ids: Tuple[int, ...] = ()
    max_position: int = 1 << 20

    @staticmethod
    def from_dict(raw: Mapping[str, Any]) -> "PoraraxConfig":
        problems = []

        def need(d, key, kind, where):
            if not isinstance(d, Mapping) or key not in d or d[key] is None:
                problems.append(f"{where}{key} is missing")
                return kind(1)
            try:
                v = kind(d[key])
            except (TypeError, ValueError):
                problems.append(f"{where}{key} = {d[key]!r} is no {kind.__name__}")
                return kind(1)
            if not v > 0:
                problems.append(f"{where}{key} = {v} must be positive")
                return kind(1)
            return v

        def grouped(m, w):
            if m.heads % m.kv_heads:
                problems.append(f"{w}heads = {m.heads} is no multiple of kv_heads = {m.kv_heads}")
            return m

        def latent(mx, w):
            owner = mx.get("kv_from")
            if owner is not None and (isinstance(owner, bool) or not isinstance(owner, int)):
                problems.append(f"{w}kv_from = {owner!r} is no layer")
                owner = None
            mask = mx.get("mask")
            return PoraraxLatent(
                heads=need(mx, "heads", int, w), dim=need(mx, "dim", int, w), vdim=need(mx, "vdim", int, w),
                kv_rank=need(mx, "kv_rank", int, w), q_rank=need(mx, "q_rank", int, w), scale=need(mx, "scale", float, w),
                window=None if mask is None else need(mask, "size", int, w + "mask."), kv_from=owner)

        def attention(mx, w):
            rot, base, dims = mx.get("rot"), None, 0
            if rot is not None and rot.get("dims") != 0:
                base, dims = need(rot, "base", float, w + "rot."), need(rot, "dims", int, w + "rot.")
            a = PoraraxAttention(heads=need(mx, "heads", int, w), kv_heads=need(mx, "kv_heads", int, w), dim=need(mx, "dim", int, w),
                                 vdim=need(mx, "vdim", int, w), scale=need(mx, "scale", float, w), rot_base=base, rot_dims=dims)
            if a.rot_dims % 2 or a.rot_dims > a.dim:
                problems.append(f"{w}rot.dims = {a.rot_dims} must be even and at most dim = {a.dim}")
            return grouped(a, w)

        def delta(mx, w):
            return grouped(PoraraxDelta(heads=need(mx, "heads", int, w), kv_heads=need(mx, "kv_heads", int, w), dim=need(mx, "dim", int, w),
                                        vdim=need(mx, "vdim", int, w), conv=need(mx, "conv", int, w)), w)

        layers = []
        raw_layers = raw.get("layers")
        if not isinstance(raw_layers, (list, tuple)) or not raw_layers:
            problems.append("layers is missing or empty")
            raw_layers = []
        readers = {"latent_attention": latent, "attention": attention, "delta": delta}
        for i, L in enumerate(raw_layers):
            w = f"layers[{i}]."
            kind = L.get("type") if isinstance(L, Mapping) else None
            if kind not in MIXER_TYPES:
                problems.append(f"{w}type = {kind!r} (known: {', '.join(MIXER_TYPES)})")
                layers.append(None)                       # (a later layer may name a layer by its place)
                continue
            mixer = readers[kind](L.get("mixer") or {}, w + "mixer.")
            mlp, rm = None, L.get("mlp")
            if rm is not None:
                wl = w + "mlp."
                if rm.get("kind", "moe") != "moe":
                    problems.append(f"{wl}kind = {rm.get('kind')!r} (known: moe)")
                else:
                    router, expert = rm.get("router"), rm.get("expert")
                    mlp = PoraraxMoe(experts=need(router, "experts", int, wl + "router."), top=need(router, "top", int, wl + "router."),
                                     ff=need(expert, "ff", int, wl + "expert."), limit=need(expert, "limit", float, wl + "expert."))
                    if mlp.top > mlp.experts:
                        problems.append(f"{wl}router.top = {mlp.top} of {mlp.experts} experts")
            layers.append(PoraraxLayer(kind, mixer, mlp))
        for i, l in enumerate(layers):
            j = l.mixer.kv_from if l is not None and l.type == "latent_attention" else None
            if j is None:
                continue
            owner = layers[j] if 0 <= j < i else None
            if owner is None or owner.type != "latent_attention" or owner.mixer.kv_from is not None:
                problems.append(f"layers[{i}].mixer.kv_from = {j} names no earlier latent_attention layer with a latent of its own")
            elif owner.mixer.kv_rank != l.mixer.kv_rank:
                problems.append(f"layers[{i}].mixer.kv_rank = {l.mixer.kv_rank}, layer {j}'s is {owner.mixer.kv_rank}")
        cfg = PoraraxConfig(
            architecture=str(raw.get("architecture", "Porarax")),
            vocab=need(raw, "vocab", int, ""), width=need(raw, "width", int, ""),
            norm_eps=need(raw.get("norm") or {}, "eps", float, "norm."), layers=tuple(layers),
            torch_dtype=str(raw.get("torch_dtype", "bfloat16")),
            eos_token_ids=tuple(int(t) for t in raw.get("eos_token_ids", ()) or ()),
            max_position=int(raw.get("max_position", 1 << 20)))
        if problems:
            raise ConfigError("config.json does not describe a Porarax model: " + "; ".join(problems))
        return cfg
