"""The Lumevik design in plain float64: one function per mechanism, whole sequences, every score written
out.  Slow on purpose; shares no code with the engine.

Notation: x [T, d] the stream, n the normed stream that a sublayer reads, W the weights by checkpoint name
(float64), positions 0 .. T-1, cfg the dict that config.json holds.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_around_zero(x, w, eps):
    """An RMS norm whose stored weight is the distance from one."""
    return unit_rms(x, eps) * (1.0 + w)


# ------------------------------------------------------------------ which keys a query reads
def seen_keys(T, window=None, keep=0):
    """[T, T] bool: query i reads key j if j <= i and the key is near (i - j < window) or among the first ``keep``."""
    i, j = torch.arange(T).view(T, 1), torch.arange(T).view(1, T)
    causal = j <= i
    return causal if window is None else causal & ((i - j < window) | (j < keep))


# ------------------------------------------------------------------ distance bias
def distance_bucket(n, B, far):
    """Row of the bias table for distance n: a row each below half of the table, then rows that widen with the
    logarithm, the last one from ``far`` on."""
    half = B // 2
    if n < half:
        return n
    return min(B - 1, half + math.floor(math.log(n / half) / math.log(far / half) * (B - half)))


def distance_bias(rel, T, far):
    """[H, T, T]: rel[bucket(i - j), h] where j <= i."""
    B, H = rel.shape
    row = torch.tensor([distance_bucket(n, B, far) for n in range(T)])
    dist = (torch.arange(T).view(T, 1) - torch.arange(T).view(1, T)).clamp(min=0)
    return rel[row[dist]].permute(2, 0, 1)


# ------------------------------------------------------------------ softmax attention
def softmax_attention(q, k, v, scale, seen, bias=None, one_more=False):
    """q [T, H, D], k [T, G, D], v [T, G, V].  score = q.k * scale + bias; with ``one_more`` the denominator is
    1 + the sum of the exponentials."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=F64)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        if bias is not None:
            s = s + bias[h]
        s = s.masked_fill(~seen, -math.inf)
        m = s.max(-1, keepdim=True).values
        if one_more:
            m = m.clamp(min=0.0)
        e = torch.exp(s - m)
        den = e.sum(-1, keepdim=True) + (torch.exp(-m) if one_more else 0.0)
        out[:, h] = (e / den) @ v[:, g]
    return out


def mixed_values(v, first, lam):
    """A layer's values blended with the ones that the first such layer formed for the same token."""
    return (1.0 - lam) * v + lam * first


def attention(n, W, p, mx, eps, carried):
    """The 'attention' mixer.  ``carried``: a dict that keeps the first mixing layer's values."""
    T = n.shape[0]
    H, G, D, V = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = (n @ W[p + "q"].T).view(T, H, D)
    k = (n @ W[p + "k"].T).view(T, G, D)
    v = (n @ W[p + "v"].T).view(T, G, V)
    if mx.get("v_mix"):
        if "v" in carried:
            v = mixed_values(v, carried["v"], W[p + "vmix"])
        else:
            carried["v"] = v
    mask = mx.get("mask") or {}
    o = softmax_attention(q, k, v, mx["scale"], seen_keys(T, mask.get("size"), mask.get("keep_first", 0)),
                          distance_bias(W[p + "rel"], T, mx["bias_max"]), one_more=True)
    return o.reshape(T, -1) @ W[p + "o"].T


def latent_attention(n, W, p, mx, eps, carried):
    """Queries through a latent of their own, keys and values expanded from a cached latent; every earlier key."""
    T, H = n.shape[0], mx["heads"]
    cq = unit_rms(n @ W[p + "dq"].T, eps) * W[p + "dq.norm"]
    q = (cq @ W[p + "uq"].T).view(T, H, mx["dim"])
    c = unit_rms(n @ W[p + "dkv"].T, eps) * W[p + "dkv.norm"]
    k = (c @ W[p + "uk"].T).view(T, H, mx["dim"])
    v = (c @ W[p + "uv"].T).view(T, H, mx["vdim"])
    o = softmax_attention(q, k, v, mx["scale"], seen_keys(T))
    return o.reshape(T, -1) @ W[p + "o"].T


# ------------------------------------------------------------------ feed-forward
def clamped_glu(h, W, p, limit):
    g = torch.clamp(h @ W[p + "gate"].T, max=limit)
    u = torch.clamp(h @ W[p + "up"].T, min=-limit, max=limit)
    return (g / (1.0 + torch.exp(-1.702 * g)) * (u + 1.0)) @ W[p + "down"].T


def open_groups(choice, count, keep):
    """[T, E] bool: experts of the ``keep`` groups whose largest choice score is largest."""
    T, E = choice.shape
    best = choice.view(T, count, E // count).max(-1).values
    order = torch.sort(best, dim=-1, descending=True, stable=True).indices[:, :keep]
    ok = torch.zeros(T, count, dtype=torch.bool).scatter_(1, order, True)
    return ok.repeat_interleave(E // count, dim=1)


def router_choice(n, W, p, router):
    """(experts [T, top], scores [T, E]): chosen by softmax score + correction inside the open groups."""
    s = torch.softmax(n @ W[p + "router"].T, dim=-1)
    c = s + W[p + "correction"]
    groups = router.get("groups")
    if groups:
        c = c.masked_fill(~open_groups(c, groups["count"], groups["keep"]), -math.inf)
    return torch.sort(c, dim=-1, descending=True, stable=True).indices[:, :router["top"]], s


def experts(n, W, p, mlp, take=None):
    chosen, s = router_choice(n, W, p, mlp["router"])
    if take is not None:
        chosen = take
    w = s.gather(1, chosen)
    w = w / (w.sum(-1, keepdim=True) + 1e-20)
    out = torch.zeros_like(n)
    for t in range(n.shape[0]):
        for j in range(chosen.shape[1]):
            out[t] += w[t, j] * clamped_glu(n[t:t + 1], W, f"{p}e{int(chosen[t, j])}.", mlp["expert"]["limit"])[0]
    if mlp.get("shared"):
        share = torch.sigmoid(n @ W[p + "shared.sg"].T)
        out = out + share * clamped_glu(n, W, p + "shared.", mlp["shared"]["limit"])
    return out, chosen


# ------------------------------------------------------------------ the model
MIXERS = {"attention": attention, "latent_attention": latent_attention}


def forward(tokens, W, cfg, take=None, streams=None, chosen=None):
    """Logits [T, vocab] of one sequence from its first token.  ``streams``: a list that receives the
    stream after every layer; ``take``: experts per layer with experts instead of the routers' choice;
    ``chosen``: a list that receives the experts taken."""
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.tensor(list(tokens))]
    carried, run = {}, 0
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + MIXERS[L["type"]](norm_around_zero(x, W[p + "norm1"], eps), W, p + "mix.", L["mixer"], eps, carried)
        mlp = L.get("mlp")
        if mlp:
            n = norm_around_zero(x, W[p + "norm2"], eps)
            if mlp["kind"] == "dense":
                x = x + clamped_glu(n, W, p + "mlp.", mlp["limit"])
            else:
                f, c = experts(n, W, p + "mlp.", mlp, None if take is None else take[run])
                x = x + f
                if chosen is not None:
                    chosen.append(c)
                run += 1
        if streams is not None:
            streams.append(x.clone())
    return norm_around_zero(x, W["final.norm"], eps) @ W["head"].T
