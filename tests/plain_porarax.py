"""The Porarax design in plain float64: one function per mechanism, whole sequences, the recurrence token by token,
every score written out.  Slow on purpose; shares no code with the engine.

Notation: x [T, d] the stream, n the normed stream that both sublayers of a layer read, W the weights by checkpoint
name (float64), positions 0 .. T-1, cfg the dict that config.json holds.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, w, eps):
    return unit_rms(x, eps) * w


def silu(z):
    return z * torch.sigmoid(z)


# ------------------------------------------------------------------ which keys a query reads
def seen_keys(T, window=None):
    """[T, T] bool: query i reads key j if j <= i and, under a window, i - j < window."""
    i, j = torch.arange(T).view(T, 1), torch.arange(T).view(1, T)
    return (j <= i) if window is None else (j <= i) & (i - j < window)


def softmax_attention(q, k, v, scale, seen):
    """q [T, H, D], k [T, G, D], v [T, G, V] -> [T, H, V]; query head h reads key/value head h // (H / G)."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=F64)
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].T) * scale).masked_fill(~seen, -math.inf)
        e = torch.exp(s - s.max(-1, keepdim=True).values)
        out[:, h] = (e / e.sum(-1, keepdim=True)) @ v[:, g]
    return out


# ------------------------------------------------------------------ attention
def turn_neighbours(x, rot):
    """x [T, heads, D]: elements (2i, 2i + 1) of the first ``dims`` turn by p * base^(-2i/dims)."""
    T, dims = x.shape[0], rot["dims"]
    f = torch.tensor([rot["base"] ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F64)
    ang = torch.arange(T, dtype=F64).view(T, 1, 1) * f
    c, s = torch.cos(ang), torch.sin(ang)
    y = x.clone()
    u, w = x[..., 0:dims:2], x[..., 1:dims:2]
    y[..., 0:dims:2], y[..., 1:dims:2] = u * c - w * s, w * c + u * s
    return y


def attention(n, W, p, mx, eps):
    """Grouped-query attention; q and k turn, then every head of them is divided by its root mean square; the heads'
    results times a sigmoid gate, element by element."""
    T = n.shape[0]
    H, G, D, V = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = (n @ W[p + "q"].T).view(T, H, D)
    k = (n @ W[p + "k"].T).view(T, G, D)
    v = (n @ W[p + "v"].T).view(T, G, V)
    if mx.get("rot"):
        q, k = turn_neighbours(q, mx["rot"]), turn_neighbours(k, mx["rot"])
    o = softmax_attention(unit_rms(q, eps), unit_rms(k, eps), v, mx["scale"], seen_keys(T))
    return (o.reshape(T, H * V) * torch.sigmoid(n @ W[p + "g"].T)) @ W[p + "o"].T


# ------------------------------------------------------------------ latent attention
def latent(n, W, p, eps):
    return norm(n @ W[p + "dkv"].T, W[p + "dkv.norm"], eps)


def latent_attention(n, W, p, mx, eps, c):
    """Queries through a latent of their own; keys and values expanded from the latent c [T, rank], this layer's or an
    earlier one's."""
    T, H = n.shape[0], mx["heads"]
    q = (norm(n @ W[p + "dq"].T, W[p + "dq.norm"], eps) @ W[p + "uq"].T).view(T, H, mx["dim"])
    k = (c @ W[p + "uk"].T).view(T, H, mx["dim"])
    v = (c @ W[p + "uv"].T).view(T, H, mx["vdim"])
    o = softmax_attention(q, k, v, mx["scale"], seen_keys(T, (mx.get("mask") or {}).get("size")))
    return o.reshape(T, -1) @ W[p + "o"].T


# ------------------------------------------------------------------ gated delta rule
def short_conv(x, w):
    """y[t, c] = sum_j w[c, j] x[t - taps + 1 + j, c], zeros before the first token."""
    T, taps = x.shape[0], w.shape[1]
    y = torch.zeros_like(x)
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            y[back:] += w[:, j] * x[:T - back]
    return y


def unit_vector(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_recurrence(q, k, v, g, beta):
    """q, k [T, H, D], v [T, H, V], g, beta [T, H].  S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q.
    Returns o [T, H, V] and the last state [H, D, V]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=F64)
    out = torch.zeros(T, H, v.shape[-1], dtype=F64)
    for t in range(T):
        S = g[t].view(H, 1, 1) * S
        u = beta[t].view(H, 1) * (v[t] - (S * k[t].unsqueeze(-1)).sum(1))
        S = S + k[t].unsqueeze(-1) * u.unsqueeze(1)
        out[t] = (S * q[t].unsqueeze(-1)).sum(1)
    return out, S


def delta_inputs(n, W, p, mx):
    """q, k, v by heads, the decays and the step sizes."""
    T = n.shape[0]
    H, G, D, V = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    row = lambda s: silu(short_conv(n @ W[p + s].T, W[p + s + ".conv"]))
    q = unit_vector(row("q").view(T, G, D)).repeat_interleave(H // G, dim=1) / math.sqrt(D)
    k = unit_vector(row("k").view(T, G, D)).repeat_interleave(H // G, dim=1)
    v = row("v").view(T, H, V)
    beta = torch.sigmoid(n @ W[p + "b"].T)
    g = torch.exp(-torch.exp(W[p + "A_log"]) * torch.nn.functional.softplus(n @ W[p + "a"].T + W[p + "dt_bias"], threshold=700))
    return q, k, v, g, beta


def delta_mixer(n, W, p, mx, eps):
    T = n.shape[0]
    o, _ = delta_recurrence(*delta_inputs(n, W, p, mx))
    y = norm(o, W[p + "norm"], eps).reshape(T, -1) * silu(n @ W[p + "g"].T)
    return y @ W[p + "o"].T


# ------------------------------------------------------------------ feed-forward
def bounded_glu(h, W, p, limit):
    g = torch.clamp(h @ W[p + "gate"].T, max=limit)
    u = torch.clamp(h @ W[p + "up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ W[p + "down"].T


def router_logits(n, W, p):
    return n @ W[p + "router"].T + W[p + "router.b"]


def experts(n, W, p, mlp, take=None):
    """(result, experts taken [T, top]); ``take``: experts to use instead of the router's own choice."""
    z = router_logits(n, W, p)
    chosen = torch.sort(z, dim=-1, descending=True, stable=True).indices[:, :mlp["router"]["top"]] if take is None else take
    w = torch.softmax(z.gather(1, chosen), dim=-1)
    out = torch.zeros_like(n)
    for e in range(z.shape[1]):
        for j in range(chosen.shape[1]):
            rows = (chosen[:, j] == e).nonzero().view(-1)
            if rows.numel():
                out[rows] += w[rows, j:j + 1] * bounded_glu(n[rows], W, f"{p}e{e}.", mlp["expert"]["limit"])
    return out, chosen


# ------------------------------------------------------------------ the model
def forward(tokens, W, cfg, take=None, streams=None, chosen=None):
    """Logits [T, vocab] of one sequence from its first token.  ``streams``: a list that receives the stream after
    every layer; ``take``: experts per layer with experts instead of the routers' choice; ``chosen``: a list that
    receives the experts taken."""
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.tensor(list(tokens))]
    latents, run = {}, 0
    for i, L in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", L["mixer"]
        n = norm(x, W[p + "norm1"], eps)
        if L["type"] == "latent_attention":
            owner = mx.get("kv_from")
            if owner is None:
                owner, latents[i] = i, latent(n, W, p + "mix.", eps)
            y = latent_attention(n, W, p + "mix.", mx, eps, latents[owner])
        else:
            y = {"attention": attention, "delta": delta_mixer}[L["type"]](n, W, p + "mix.", mx, eps)
        mlp = L.get("mlp")
        if mlp:
            f, c = experts(n, W, p + "mlp.", mlp, None if take is None else take[run])
            y = y + f
            if chosen is not None:
                chosen.append(c)
            run += 1
        x = x + y
        if streams is not None:
            streams.append(x.clone())
    return norm(x, W["final.norm"], eps) @ W["embed"].T
