"""The gated delta rule: a recurrent state per head that every token corrects.

Per value head, with unit vectors k and q (q times ``key_dim``^-1/2) of the q/k head that it shares with its neighbours, a
decay g and a step size beta of its own:

    S <- g S,   u = beta (v - S^T k),   S <- S + k u^T,   o = S^T q

so a token writes what its value differs from what the state already holds under its key.  q, k and v are projections that
pass a short causal convolution over time per channel and silu (``*_conv`` [channels, taps], the last column the token's
own); q and k heads then become x / sqrt(sum x^2 + 1e-6).  beta = sigmoid(W_b x), g = exp(-exp(a_log) softplus(W_a x +
dt_bias)).  Every head's o is RMS-normed over its values with one weight vector for all heads and multiplied with
silu(W_g x), then the output projection.

The state S and the convolution's last taps - 1 inputs are kept between steps in two state tensors (``state`` and
``conv``).  Unit vectors, decays, step sizes, the recurrence and the norm are fp32 in both dtypes; projections and the
convolution's results take the run's dtype.
"""
from __future__ import annotations

import numpy as np
import torch

from .base import Mixer, ParamSpec, CacheNeed, StateNeed, register, register_step_array
from .linear import linear, Weight
from ..csrc import hipops

UNIT_EPS = 1e-6      # under the root of a unit vector's length


def _chunks(host):
    """The step's tokens in chunks for the matrix-unit kernel; a step of single tokens runs without them."""
    if int(host.counts.max(initial=1)) <= 1:
        return np.zeros(0, dtype=np.int32), 0
    return hipops.delta_chunks(host.counts, host.cu_seqlens)


CHUNKS = "delta_rule.chunks"
register_step_array(CHUNKS, _chunks)


@register("mixer", "delta_rule")
class DeltaRule(Mixer):
    graph_safe = True

    def __init__(self, env, hidden_size, n_heads, n_qk_heads, key_dim, value_dim, conv_taps, norm_eps):
        self.env = env
        self.d, self.H, self.G = int(hidden_size), int(n_heads), int(n_qk_heads)
        self.D, self.V, self.taps, self.eps = int(key_dim), int(value_dim), int(conv_taps), float(norm_eps)
        if self.H % self.G:
            raise ValueError(f"delta_rule: {self.H} heads over {self.G} heads of q and k")
        if self.D > 256:
            raise ValueError(f"delta_rule: {self.D} key channels a head (at most 256)")
        if not 1 <= self.taps <= 32:
            raise ValueError(f"delta_rule: a convolution of {self.taps} taps (1 to 32)")
        self.n_conv = 2 * self.G * self.D + self.H * self.V
        self.mfma = hipops.delta_chunk_ok(env.dtype, self.G, self.H, self.D, self.V)
        self.step_arrays = (CHUNKS,) if self.mfma else ()
        self.w_in = self.w_conv = self.a_log = self.dt_bias = self.w_norm = self.wo = None

    # ------------------------------------------------------------------ tensors
    def params(self):
        d, H, GD, HV = self.d, self.H, self.G * self.D, self.H * self.V
        p = {"q_proj": ParamSpec((GD, d)), "k_proj": ParamSpec((GD, d)), "v_proj": ParamSpec((HV, d)),
             "gate_proj": ParamSpec((HV, d)), "a_proj": ParamSpec((H, d)), "b_proj": ParamSpec((H, d)), "o_proj": ParamSpec((d, HV)),
             "a_log": ParamSpec((H,), kind="vector", init="normal"), "dt_bias": ParamSpec((H,), kind="vector", init="normal"),
             "norm": ParamSpec((self.V,), kind="vector", init="ones")}
        for name, n in (("q_conv", GD), ("k_conv", GD), ("v_conv", HV)):
            p[name] = ParamSpec((n, self.taps), kind="vector", init="normal")
        return p

    def load(self, t):
        # one product for everything that reads the mixer's input: [q | k | v | gate | a | b]
        mats = [t[k] for k in ("q_proj", "k_proj", "v_proj", "gate_proj", "a_proj", "b_proj")]
        dts = {m.dtype for m in mats}
        dt = torch.float32 if len(dts) > 1 else dts.pop()
        w = torch.cat([m.to(dt) for m in mats], dim=0)
        pad = -w.shape[0] % 16               # whole bands of 16 rows: the weight can be kept in operand order
        if pad:
            w = torch.cat([w, torch.zeros((pad, w.shape[1]), dtype=dt, device=w.device)], dim=0)
        self.w_in = Weight(w)
        # tap by tap, [taps, channels]: the kernel's loads of one tap are consecutive
        self.w_conv = torch.cat([t["q_conv"], t["k_conv"], t["v_conv"]], dim=0).float().t().contiguous()
        self.a_log, self.dt_bias = t["a_log"].float().contiguous(), t["dt_bias"].float().contiguous()
        self.w_norm = t["norm"].float().contiguous()
        self.wo = Weight(t["o_proj"])

    def slow_paths(self, page_size):
        notes = []
        if self.env.dtype == torch.bfloat16 and self.w_in is not None:
            if not self.mfma:
                notes.append(f"the delta rule runs token by token: {self.D} key channels a head in rows of {self.n_conv} (the matrix-unit kernel "
                             f"takes 32, 64, 96 or 128 in rows of a multiple of 8)")
            notes += self.w_in.slow_reason("input projection") + self.wo.slow_reason("output projection")
        return notes

    def cache_needs(self):
        needs = {"state": CacheNeed(state=StateNeed((self.H, self.D, self.V), torch.float32))}
        if self.taps > 1:
            needs["conv"] = CacheNeed(state=StateNeed((self.taps - 1, self.n_conv), torch.float32))
        return needs

    # ------------------------------------------------------------------ the step
    def forward(self, x, ctx, cache):
        T, ws = x.shape[0], ctx.ws
        H, G, D, V = self.H, self.G, self.D, self.V
        GD, HV, n = G * D, H * V, self.n_conv
        state = (cache["state"] if isinstance(cache, dict) else cache).state
        proj = ws.take((T, self.w_in.shape[0]), x.dtype)
        linear(x, self.w_in, proj, ws=ws)
        qkv = ws.take((T, n), x.dtype)
        hipops.causal_conv(proj[:, :n], self.w_conv, qkv, cache["conv"].state if self.taps > 1 else None, ctx.seq_of_token,
                           ctx.cu_seqlens, ctx.seq_slots, act="silu")
        q, k, v = qkv[:, :GD], qkv[:, GD:2 * GD], qkv[:, 2 * GD:]
        qk_scale, gates = ws.take((T, 2, G), torch.float32), ws.take((T, 2, H), torch.float32)
        hipops.delta_gates(q, k, proj[:, n + HV:n + HV + H], proj[:, n + HV + H:n + HV + 2 * H], self.a_log, self.dt_bias, qk_scale, gates,
                           G, H, D, q_scale=float(D) ** -0.5, eps=UNIT_EPS)
        o = ws.take((T, HV), torch.float32)
        if self.mfma and not ctx.decode_only:
            chunks, n_chunks = ctx.derived[CHUNKS]
            scratch = ws.take((hipops.delta_chunk_workspace(n_chunks, G, H, D),), torch.uint8)
            hipops.delta_chunk(q, k, v, qk_scale, gates, state, o, chunks, n_chunks, ctx.seq_slots, ctx.n_seqs, scratch, G, H, D, V)
        else:
            hipops.delta_scan(q, k, v, qk_scale, gates, state, o, ctx.cu_seqlens, ctx.seq_slots, ctx.n_seqs, G, H, D, V, single=ctx.decode_only)
        y = ws.take((T, HV), x.dtype)
        hipops.gated_group_norm(o, self.w_norm, y, V, self.eps, gate=proj[:, n:n + HV], act="silu")
        out = ws.take((T, self.d), torch.float32)
        linear(y, self.wo, out, ws=ws)
        return out
