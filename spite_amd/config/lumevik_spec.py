"""A Lumevik model as a list of parts.

Every layer is a ``prenorm`` block under RMS norms whose weights are stored around zero.  Mixers: ``attention`` is
``wide_attention`` with a bias by distance (``distance_buckets``), a window with kept first positions, a sink of score
zero and blended values; ``latent_attention`` is the part of that name with a latent for the queries and no rotated
part.  Feed-forward: ``dense_glu`` or ``moe_topk_sigmoid`` with softmax scores, groups of experts and a gated shared
expert, both with the clamped gate.  Tensor names: ``l<i>.norm1|norm2``, ``.mix.q|k|v|rel|vmix|o`` or
``.mix.dq|dq.norm|uq|dkv|dkv.norm|uk|uv|o``, ``.mlp.gate|up|down`` or ``.mlp.router|correction|e<k>.*|shared.*``;
``embed``, ``final.norm``, ``head``.
"""
from __future__ import annotations

from .lumevik import LumevikConfig, LumevikDense
from .registry import register_architecture
from ..parts.base import PartSpec, BlockSpec, LayerCall, ModelSpec


def _norm(cfg, name):
    return PartSpec("rms", {"width": cfg.width, "eps": cfg.norm_eps, "offset": 1.0}, {"weight": name})


def _mixer(cfg, layer, p):
    mx = layer.mixer
    if layer.type == "attention":
        names = {f"{s}_proj": p + s for s in "qkvo"}
        names["rel"] = p + "rel"
        if mx.v_mix:
            names["v_mix"] = p + "vmix"
        return PartSpec("wide_attention", dict(
            hidden_size=cfg.width, n_heads=mx.heads, n_kv_heads=mx.kv_heads, key_dim=mx.dim, value_dim=mx.vdim, scale=mx.scale,
            visibility="full" if mx.window is None else "window", span=mx.window or 0,
            keep=mx.keep_first if mx.window is not None else 0, sinks="zero",
            score_position=PartSpec("distance_buckets", {"n_heads": mx.heads, "far": mx.bias_max}),
            value_blend="values" if mx.v_mix else None), names)
    names = {"q": p + "uq"}
    names.update({k: p + k for k in ("dq", "dq.norm", "dkv", "dkv.norm", "uk", "uv", "o")})
    return PartSpec("latent_attention", dict(
        hidden_size=cfg.width, n_heads=mx.heads, dim=mx.dim, rot_dim=0, v_dim=mx.vdim, kv_rank=mx.kv_rank, q_rank=mx.q_rank,
        scale=mx.scale, position=None, norm_eps=cfg.norm_eps), names)


def _ffn(cfg, ml, p):
    if isinstance(ml, LumevikDense):
        return PartSpec("dense_glu", dict(hidden_size=cfg.width, intermediate_size=ml.ff, activation="clamped", limit=ml.limit),
                        {f"{k}_proj": p + k for k in ("gate", "up", "down")})
    names = {k: p + k for k in ("router", "correction")}
    for e in range(ml.experts):
        names.update({f"e{e}.{k}": f"{p}e{e}.{k}" for k in ("gate", "up", "down")})
    if ml.shared is not None:
        names.update({f"shared.{k}": f"{p}shared.{k}" for k in ("gate", "up", "down", "sg")})
    return PartSpec("moe_topk_sigmoid", dict(
        hidden_size=cfg.width, intermediate_size=ml.expert.ff, n_experts=ml.experts, top_k=ml.top,
        shared_intermediate_size=None if ml.shared is None else ml.shared.ff, score_bias=True, renormalize=True,
        scoring="softmax", groups=ml.groups, activation="clamped", limit=ml.expert.limit,
        shared_limit=None if ml.shared is None else ml.shared.limit, shared_gate=ml.shared is not None), names)


def build_spec(cfg: LumevikConfig) -> ModelSpec:
    blocks = []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        has = layer.mlp is not None
        blocks.append(BlockSpec("prenorm", _norm(cfg, p + "norm1"), _mixer(cfg, layer, p + "mix."),
                                _norm(cfg, p + "norm2") if has else None, _ffn(cfg, layer.mlp, p + "mlp.") if has else None))
    return ModelSpec(
        architecture=cfg.architecture, vocab_size=cfg.vocab, hidden_size=cfg.width, blocks=blocks,
        order=[LayerCall(block=i, cache=i) for i in range(len(blocks))], final_norm=_norm(cfg, "final.norm"),
        embed_name="embed", head_name="head", eos_token_ids=cfg.eos_token_ids, max_position=cfg.max_position, strip_prefixes=())


register_architecture("Lumevik", LumevikConfig.from_dict, build_spec)
