"""A Porarax model as a list of parts.

Every layer is a ``parallel`` block with one RMS norm: mixer and feed-forward both read norm1(x) and join the stream
together.  Mixers: ``latent_attention`` with a latent for the queries, no rotated part and a window (a layer with
``kv_from`` reads the cache of the layer it names; that layer's cache keeps what the widest of its readers needs);
``attention`` is ``wide_attention`` with a rotation of adjacent pairs, unit norms per head and a gate per element;
``delta`` is ``delta_rule``.  Feed-forward: ``moe_topk_softmax`` with a bias inside the router's logits and the clamped
gate.  The head is the embedding's table.  Tensor names: ``l<i>.norm1``, ``.mix.dq|dq.norm|uq|dkv|dkv.norm|uk|uv|o``,
``.mix.q|k|v|g|o`` and, for ``delta``, ``.mix.q.conv|k.conv|v.conv|a|b|A_log|dt_bias|norm``,
``.mlp.router|router.b|e<k>.gate|up|down``; ``embed``, ``final.norm``.
"""
from __future__ import annotations

from .porarax import PoraraxConfig
from .registry import register_architecture
from ..parts.base import PartSpec, BlockSpec, LayerCall, ModelSpec


def _reach(layers):
    """{layer that owns a latent: the widest window of the layers that read it (None: every earlier key)}."""
    reach = {}
    for i, layer in enumerate(layers):
        if layer.type != "latent_attention":
            continue
        owner, w = i if layer.mixer.kv_from is None else layer.mixer.kv_from, layer.mixer.window
        reach[owner] = w if owner not in reach else None if w is None or reach[owner] is None else max(reach[owner], w)
    return reach


def _mixer(cfg, layer, p, reach):
    mx, d, eps = layer.mixer, cfg.width, cfg.norm_eps
    if layer.type == "latent_attention":
        own = mx.kv_from is None
        names = {"q": p + "uq"}
        names.update({k: p + k for k in ("dq", "dq.norm", "uk", "uv", "o") + (("dkv", "dkv.norm") if own else ())})
        kind = lambda w: ("full" if w is None else "window", w or 0)
        (vis, span), (keep_vis, keep_span) = kind(mx.window), kind(reach)
        return PartSpec("latent_attention", dict(
            hidden_size=d, n_heads=mx.heads, dim=mx.dim, rot_dim=0, v_dim=mx.vdim, kv_rank=mx.kv_rank, q_rank=mx.q_rank, scale=mx.scale,
            position=None, norm_eps=eps, visibility=vis, span=span, own_kv=own, cache_visibility=keep_vis, cache_span=keep_span), names)
    names = {f"{s}_proj": p + s for s in "qkvo"}
    names["gate_proj"] = p + "g"
    if layer.type == "attention":
        position = None
        if mx.rot_dims:
            position = PartSpec("rotary", {"head_dim": mx.rot_dims, "theta": mx.rot_base, "pairing": "adjacent", "rotary_dim": mx.rot_dims})
        return PartSpec("wide_attention", dict(
            hidden_size=d, n_heads=mx.heads, n_kv_heads=mx.kv_heads, key_dim=mx.dim, value_dim=mx.vdim, scale=mx.scale,
            position=position, head_norm="unit", norm_eps=eps, head_gate="elements"), names)
    names.update({f"{s}_conv": f"{p}{s}.conv" for s in "qkv"})
    names.update({"a_proj": p + "a", "b_proj": p + "b", "a_log": p + "A_log", "dt_bias": p + "dt_bias", "norm": p + "norm"})
    return PartSpec("delta_rule", dict(hidden_size=d, n_heads=mx.heads, n_qk_heads=mx.kv_heads, key_dim=mx.dim, value_dim=mx.vdim,
                                       conv_taps=mx.conv, norm_eps=eps), names)


def _ffn(cfg, ml, p):
    names = {"router": p + "router", "correction": p + "router.b"}
    for e in range(ml.experts):
        names.update({f"e{e}.{k}": f"{p}e{e}.{k}" for k in ("gate", "up", "down")})
    return PartSpec("moe_topk_softmax", dict(hidden_size=cfg.width, intermediate_size=ml.ff, n_experts=ml.experts, top_k=ml.top,
                                             activation="clamped", limit=ml.limit, logit_bias=True), names)


def build_spec(cfg: PoraraxConfig) -> ModelSpec:
    norm = lambda name: PartSpec("rms", {"width": cfg.width, "eps": cfg.norm_eps}, {"weight": name})
    reach = _reach(cfg.layers)
    blocks, order = [], []
    for i, layer in enumerate(cfg.layers):
        p, owner = f"l{i}.", i
        if layer.type == "latent_attention" and layer.mixer.kv_from is not None:
            owner = layer.mixer.kv_from
        blocks.append(BlockSpec("parallel", norm(p + "norm1"), _mixer(cfg, layer, p + "mix.", reach.get(owner)), None,
                                None if layer.mlp is None else _ffn(cfg, layer.mlp, p + "mlp.")))
        cache = 2 * owner
        if layer.type == "delta" and layer.mixer.conv > 1:
            cache = {"state": cache, "conv": cache + 1}
        order.append(LayerCall(block=i, cache=cache, write=owner == i))
    return ModelSpec(
        architecture=cfg.architecture, vocab_size=cfg.vocab, hidden_size=cfg.width, blocks=blocks, order=order,
        final_norm=norm("final.norm"), embed_name="embed", head_name=None, eos_token_ids=cfg.eos_token_ids,
        max_position=cfg.max_position, strip_prefixes=())


register_architecture("Porarax", PoraraxConfig.from_dict, build_spec)
