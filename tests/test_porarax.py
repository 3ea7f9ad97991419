"""The Porarax design in the engine against the plain implementation (``plain_porarax``): every mechanism's kernel alone,
whole prompts, decoding through the cache and the recurrent state, portions down to two tokens, mixed batches with pages
and slots used again, window edges of a latent's owner and of its readers, far keys, far tokens in the state, generation."""
from __future__ import annotations

import copy
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import helpers as H
import plain_porarax as plain


# ------------------------------------------------------------------------------------------ configurations
def _latent(heads, dim, vdim, kv_rank, q_rank, scale, window=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale}
    if window is not None:
        m["mask"] = {"size": window}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return "latent_attention", m


def _attention(heads, kv, dim, vdim, scale, base=None, dims=0):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale}
    if dims:
        m["rot"] = {"base": base, "dims": dims}
    return "attention", m


def _delta(heads, kv, dim, vdim, conv):
    return "delta", {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}


def _moe(experts, top, ff, limit):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff, "limit": limit}}


def _layer(mixer, mlp):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": mlp}


# odd sizes that no fast kernel takes; all mixers, readers with a wider and a narrower window than the latent's owner, a layer
# without feed-forward, attention without rotation
SMALL = {"architecture": "Porarax", "vocab": 90, "width": 40, "norm": {"eps": 1e-5},
         "layers": [_layer(_delta(4, 2, 12, 10, 4), _moe(5, 2, 12, 0.8)),
                    _layer(_latent(3, 10, 6, 20, 14, 0.35, window=11), _moe(4, 1, 20, 0.5)),
                    _layer(_attention(4, 2, 12, 10, 0.3, 1000.0, 6), None),
                    _layer(_latent(2, 14, 9, 20, 30, 0.25, window=17, kv_from=1), _moe(3, 3, 8, 1.2)),
                    _layer(_delta(3, 3, 7, 5, 1), _moe(6, 3, 10, 0.6)),
                    _layer(_latent(4, 6, 5, 20, 9, 0.4, window=5, kv_from=1), None),
                    _layer(_attention(3, 1, 9, 14, 0.5), _moe(2, 1, 16, 2.0))]}
# sizes that the matrix-unit kernels take in bfloat16
WIDE = {"architecture": "Porarax", "vocab": 320, "width": 128, "norm": {"eps": 1e-6},
        "layers": [_layer(_latent(5, 64, 32, 96, 64, 0.125), _moe(8, 2, 64, 1.0)),
                   _layer(_delta(4, 2, 64, 48, 4), _moe(12, 3, 32, 0.9)),
                   _layer(_attention(8, 2, 128, 64, 0.09, 5000.0, 32), _moe(4, 1, 64, 1.4)),
                   _layer(_latent(16, 32, 64, 96, 128, 0.17, window=50, kv_from=0), None),
                   _layer(_delta(2, 1, 128, 80, 2), _moe(6, 2, 96, 0.7)),
                   _layer(_attention(2, 2, 48, 64, 0.14, 20000.0, 48), _moe(8, 4, 32, 1.1))]}
# values that are 1 or equal where the other configurations have them apart
ONES = {"architecture": "Porarax", "vocab": 50, "width": 24, "norm": {"eps": 1e-3},
        "layers": [_layer(_delta(1, 1, 1, 1, 1), _moe(1, 1, 8, 1.0)),
                   _layer(_latent(1, 1, 1, 1, 1, 1.0, window=1), _moe(2, 2, 1, 0.1)),
                   _layer(_attention(1, 1, 2, 1, 1.0, 10.0, 2), None),
                   _layer(_latent(4, 4, 4, 1, 4, 0.5, window=2, kv_from=1), _moe(3, 1, 4, 1.0)),
                   _layer(_delta(4, 4, 4, 4, 4), None)]}
CONFIGS = {"small": SMALL, "wide": WIDE, "ones": ONES}
PAGE = {"small": 16, "wide": 32, "ones": 4}
LENGTHS = {"small": [1, 45, 23, 60, 2, 31, 17], "wide": [90, 1, 140, 33, 75], "ones": [30, 1, 44, 9]}


def planted(cfg, seed, gain=3.0, std=0.08):
    """Random tensors with sharper attention, decays and step sizes over their whole range, convolutions whose taps all
    count, routers that tell experts apart and biases that change choices, gates that reach their limits."""
    from spite_amd.weights.random_init import random_tensors
    t = random_tensors(cfg, seed, std)
    g = torch.Generator().manual_seed(seed)
    rnd = lambda shape, s=1.0: torch.randn(shape, generator=g) * s
    t["embed"] = t["embed"] * (0.7 / std)
    for name in sorted(t):
        if name.endswith("norm1") or name.endswith(".norm"):
            t[name] = 1.0 + rnd(t[name].shape, 0.3)
        elif name.endswith((".gate", ".up")):
            t[name] = t[name] * 1.5
        elif name.endswith(".conv"):
            t[name] = rnd(t[name].shape, 0.6)
        elif name.endswith("A_log"):
            t[name] = rnd(t[name].shape, 1.0) - 1.0
        elif name.endswith("dt_bias"):
            t[name] = rnd(t[name].shape, 1.0)
        elif name.endswith(("mix.a", "mix.b", "mix.g")):
            t[name] = t[name] * 4.0
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}.mix."
        if L["type"] == "attention":
            t[p + "q"] = t[p + "q"] * gain
        elif L["type"] == "latent_attention":
            t[p + "uq"], t[p + "uk"] = t[p + "uq"] * gain, t[p + "uk"] * gain
        else:
            for s in "qkv":
                t[p + s] = t[p + s] * 4.0
        if L["mlp"]:
            t[f"l{i}.mlp.router"] = t[f"l{i}.mlp.router"] * 6.0
            t[f"l{i}.mlp.router.b"] = rnd((L["mlp"]["router"]["experts"],), 0.5)
    return t


def make_model(folder, cfg, seed, dtype, **kw):
    from spite_amd.weights.random_init import write_random_model
    write_random_model(str(folder), cfg, seed, dtype=dtype, overrides=planted(cfg, seed, **kw))
    return H.read_weights(str(folder))


def requests(vocab, lengths, seed):
    return {f"r{i}": H.random_tokens(vocab, n, seed + 13 * i) for i, n in enumerate(lengths)}


def tops(cfg):
    return [L["mlp"]["router"]["top"] for L in cfg["layers"] if L["mlp"]]


def plain_rows(cfg, weights, reqs, taken=None, chosen=None):
    """{(request, position): logits}; ``taken``: {request: [experts [T, top] per layer with experts]}; ``chosen`` receives them."""
    rows = {}
    for rid, toks in reqs.items():
        got = []
        out = plain.forward(toks, weights, cfg, take=None if taken is None else taken[rid], chosen=got).to(torch.float32).numpy()
        if chosen is not None:
            chosen[rid] = got
        for i in range(len(toks)):
            rows[(rid, i)] = out[i]
    return rows


def experts_of(cfg, steps, routing):
    """{request: [experts [T, top] per layer with experts]} from what a replay recorded step by step."""
    tk, parts = tops(cfg), {}
    for rec in steps:
        off = 0
        for e in rec["entries"]:
            n = len(e["tokens"])
            for k, top in enumerate(tk):
                parts.setdefault(e["id"], [[] for _ in tk])[k].append(np.asarray(routing[rec["step"]][k]).reshape(-1, top)[off:off + n])
            off += n
    return {rid: [torch.from_numpy(np.concatenate(v).astype(np.int64)) for v in per] for rid, per in parts.items()}


def experts_for(cfg, steps, experts):
    """{step: [experts of the step's tokens, one array per layer with experts]}: ``experts`` cut as ``steps`` cuts."""
    n_runs, fed, take = len(tops(cfg)), {}, {}
    for rec in steps:
        per = [[] for _ in range(n_runs)]
        for e in rec["entries"]:
            at, n = fed.get(e["id"], 0), len(e["tokens"])
            for k in range(n_runs):
                per[k].append(experts[e["id"]][k][at:at + n].numpy())
            fed[e["id"]] = at + n
        take[rec["step"]] = [np.concatenate(x).astype(np.int32) if x else np.zeros((0,), np.int32) for x in per]
    return take


def engine(folder, dtype, name, **kw):
    from spite_amd import Engine
    kw.setdefault("page_size", PAGE[name])
    kw.setdefault("cache_tokens", 1024)
    kw.setdefault("max_requests", 4)
    return Engine(str(folder), dtype=dtype, device="cuda:0", **kw)


def poison(eng):
    """Every cache row and every state row holds NaN until it is written or handed out."""
    for g in eng.cache.groups:
        for half in g.halves():
            if half is not None and half.numel():
                half.fill_(float("nan"))
    for st in eng.cache.states.values():
        st.fill_(float("nan"))


def close_in_16_bits(rows, ref, scale, tol):
    """bfloat16 against the plain implementation: every row within 4 ``tol``, all but one in fifty within ``tol``."""
    over = lambda limit: [k for k in rows if not float(np.max(np.abs(rows[k].astype(np.float64) - ref[k].astype(np.float64)))) <= limit]
    far, near = over(4 * tol * scale), over(tol * scale)
    assert not far and len(near) <= max(1, len(rows) // 50), f"{len(near)} of {len(rows)} rows over {tol * scale}, {far[:3]} far over (scale {scale})"


def scale_of(rows):
    return max(float(np.abs(v).max()) for v in rows.values())


# ------------------------------------------------------------------------------------------ without a GPU
def _model(cfg):
    from spite_amd.config import read_config
    from spite_amd.engine.model import Model
    from spite_amd.engine.context import Env
    arch, typed = read_config(cfg)
    return arch, typed, Model(arch.build_spec(typed), Env(torch.float32, torch.device("cpu")))


def test_registry_and_tensor_names():
    from spite_amd.config.porarax import PoraraxConfig
    arch, cfg, model = _model(SMALL)
    assert arch.name == "Porarax" and isinstance(cfg, PoraraxConfig)
    assert cfg.layers[3].mixer.kv_from == 1 and cfg.layers[1].mixer.window == 11 and cfg.layers[0].mixer.conv == 4
    assert cfg.layers[2].mlp is None and cfg.layers[3].mlp.top == 3 and cfg.layers[6].mixer.rot_base is None
    names = {n: ps.shape for n, ps, _, _ in model.tensor_plan()}
    assert {"embed", "final.norm", "l0.norm1", "l0.mix.q.conv", "l0.mix.A_log", "l0.mix.dt_bias", "l0.mix.a", "l0.mix.b", "l0.mix.norm",
            "l1.mix.dq", "l1.mix.dq.norm", "l1.mix.dkv", "l1.mix.dkv.norm", "l1.mix.uk", "l2.mix.g", "l3.mix.dq", "l0.mlp.router.b",
            "l0.mlp.e4.down"} <= set(names)
    for absent in ("head", "l3.mix.dkv", "l3.mix.dkv.norm", "l0.norm2", "l2.mlp.router", "l2.mix.q.norm", "l0.mlp.shared.up"):
        assert absent not in names, absent
    assert names["l0.mix.q"] == (24, 40) and names["l0.mix.v"] == (40, 40) and names["l0.mix.v.conv"] == (40, 4) and names["l0.mix.g"] == (40, 40)
    assert names["l2.mix.q"] == (48, 40) and names["l2.mix.v"] == (20, 40) and names["l2.mix.g"] == (40, 40) and names["l2.mix.o"] == (40, 40)
    assert names["l3.mix.uq"] == (28, 30) and names["l3.mix.uk"] == (28, 20) and names["l0.mix.norm"] == (10,) and names["l0.mix.b"] == (4, 40)
    needs = model.cache_needs()
    assert needs[0].state.shape == (4, 12, 10) and needs[1].state.shape == (3, 88) and needs[0].kv is None
    assert needs[8].state.shape == (3, 7, 5) and (len(needs) <= 9 or needs[9] is None)       # one tap: no inputs to remember
    # the owner's cache keeps what the widest of its readers needs
    assert (needs[2].kv.visibility, needs[2].kv.span, needs[2].kv.head_dim, needs[2].kv.value_dim) == ("window", 17, 20, 0)
    assert needs[6] is None and needs[10] is None and needs[4].kv.visibility == "full"
    wide = _model(WIDE)[2].cache_needs()
    assert wide[0].kv.visibility == "full" and wide[0].kv.head_dim == 96


def test_config_errors_are_collected():
    from spite_amd.config import read_config, ConfigError
    bad = copy.deepcopy(SMALL)
    del bad["vocab"]
    bad["layers"][0]["mixer"]["kv_heads"] = 3
    bad["layers"][0]["mlp"]["router"]["top"] = 9
    bad["layers"][1]["mlp"]["expert"]["limit"] = 0.0
    bad["layers"][2]["mixer"]["rot"]["dims"] = 5
    bad["layers"][3]["mixer"]["kv_rank"] = 21
    bad["layers"][4]["mixer"]["conv"] = 0
    bad["layers"][5]["mixer"]["kv_from"] = 6
    bad["layers"][6]["type"] = "other"
    with pytest.raises(ConfigError) as e:
        read_config(bad)
    msg = str(e.value)
    for word in ("vocab", "kv_heads", "router.top = 9", "limit", "rot.dims", "kv_rank = 21", "conv", "kv_from = 6", "type"):
        assert word in msg, word
    for wrong in (3, 5, 2, -1, "1", 4):
        bad = copy.deepcopy(SMALL)
        bad["layers"][5]["mixer"]["kv_from"] = wrong                # a reader, itself, another mixer, no layer at all
        with pytest.raises(ConfigError, match="kv_from"):
            read_config(bad)


def test_plain_mechanisms():
    f64 = torch.float64
    seen = plain.seen_keys(5, 2)
    assert seen[4].tolist() == [False, False, False, True, True] and torch.equal(plain.seen_keys(4), torch.tril(torch.ones(4, 4)).bool())
    # neighbours turn, the rest passes
    x = torch.zeros(3, 1, 5, dtype=f64)
    x[:, :, 2], x[:, :, 4] = 1.0, 7.0
    y = plain.turn_neighbours(x, {"base": 16.0, "dims": 4})
    assert abs(float(y[2, 0, 2]) - math.cos(2 * 0.25)) < 1e-12 and abs(float(y[2, 0, 3]) - math.sin(2 * 0.25)) < 1e-12 and float(y[2, 0, 4]) == 7.0
    # the convolution's last column is the token's own
    c = plain.short_conv(torch.tensor([[1.0], [2.0], [4.0]], dtype=f64), torch.tensor([[100.0, 10.0, 1.0]], dtype=f64))
    assert c.view(-1).tolist() == [1.0, 12.0, 124.0]
    # the recurrence: a key written twice with step size 1 holds the second value; a key across it is left alone
    k = torch.tensor([[1.0, 0.0], [0.0, 1.0], [1.0, 0.0]], dtype=f64).view(3, 1, 2)
    v = torch.tensor([3.0, 5.0, 11.0], dtype=f64).view(3, 1, 1)
    one = torch.ones(3, 1, dtype=f64)
    o, S = plain.delta_recurrence(k, k, v, one, one)
    assert o.view(-1).tolist() == [3.0, 5.0, 11.0] and S.view(-1).tolist() == [11.0, 5.0]
    # with a decay and half a step: g S, then the correction from the decayed state, then the read
    o, S = plain.delta_recurrence(k, 2 * k, v, 0.5 * one, 0.5 * one)
    s0 = 2 * 0.5 * 3.0
    s0 = 0.25 * s0 + 2 * 0.5 * (11.0 - 2 * 0.25 * s0)
    assert abs(float(S[0, 0, 0]) - s0) < 1e-12 and abs(float(o[2]) - s0) < 1e-12
    # the gate with bounds
    W = {"gate": torch.tensor([[2.0], [-3.0]], dtype=f64), "up": torch.tensor([[-5.0], [0.2]], dtype=f64), "down": torch.eye(2, dtype=f64)}
    y = plain.bounded_glu(torch.ones(1, 1, dtype=f64), W, "", 0.5)
    assert abs(float(y[0, 0]) - 0.5 / (1 + math.exp(-1.702 * 0.5)) * 0.5) < 1e-12
    assert abs(float(y[0, 1]) - -3.0 / (1 + math.exp(1.702 * 3.0)) * 1.2) < 1e-12
    # the router's bias counts in the choice and in the weights
    W = {"router": torch.eye(3, dtype=f64), "router.b": torch.tensor([0.0, 0.0, 2.0], dtype=f64)}
    for e in range(3):
        W.update({f"e{e}.gate": torch.full((1, 3), 50.0, dtype=f64), f"e{e}.up": torch.zeros(1, 3, dtype=f64), f"e{e}.down": torch.full((3, 1), float(e), dtype=f64)})
    out, took = plain.experts(torch.tensor([[1.0, 0.5, -0.2]], dtype=f64), W, "", {"router": {"top": 2}, "expert": {"limit": 1.0}})
    w = math.exp(1.8) / (math.exp(1.8) + math.exp(1.0))
    assert took[0].tolist() == [2, 0] and abs(float(out[0, 0]) - 2 * w / (1 + math.exp(-1.702))) < 1e-12


def test_chunk_lists():
    from spite_amd.csrc import hipops
    counts = [1, 70, 32, 2, 33]
    cu = np.concatenate([[0], np.cumsum(counts)])
    arr, n = hipops.delta_chunks(counts, cu)
    first, t0, length = arr[:6], arr[6:6 + n], arr[6 + n:]
    assert n == 8 and first.tolist() == [0, 1, 4, 5, 6, 8] and length.tolist() == [1, 32, 32, 6, 32, 2, 32, 1]
    assert t0.tolist() == [0, 1, 33, 65, 71, 103, 105, 137] and arr.dtype == np.int32 and len(length) == n


# ------------------------------------------------------------------------------------------ kernels alone
def _delta_case(lens, G, Hh, D, V, dtype, seed, kind="random"):
    """Rows of a step and the plain implementation's inputs.  ``kind``: ``random``; ``same`` (all keys of a request alike, step
    sizes near 1, no decay: a chunk's triangular system is as far from the identity as it gets); ``resets`` (decays from
    1 to e^-3000 between neighbours)."""
    g = torch.Generator().manual_seed(seed)
    dt = getattr(torch, dtype)
    T = sum(lens)
    rnd = lambda *s: torch.randn(*s, generator=g)
    q, k, v = rnd(T, G * D), rnd(T, G * D), rnd(T, Hh * V)
    a, b = rnd(T, Hh) * 2, rnd(T, Hh) * 2
    a_log, dt_bias = rnd(Hh) - 1.0, rnd(Hh)
    if kind == "same":
        k = k[:1].expand(T, -1) + 0.02 * rnd(T, G * D)
        b, a = b.abs() * 2 + 4.0, a - 14.0
    elif kind == "resets":
        a = torch.where(rnd(T, Hh) > 0.8, torch.full((T, Hh), 1000.0), a - 6.0)
        a_log = torch.full((Hh,), 1.0)
    row = torch.cat([q, k, v, a, b], dim=1).to(dt)
    n = 2 * G * D
    q, k, v, a, b = (x.double() for x in row.split([G * D, G * D, Hh * V, Hh, Hh], dim=1))
    rep = Hh // G
    spread = lambda x: plain.unit_vector(x.view(T, G, D)).repeat_interleave(rep, dim=1)
    decay = torch.exp(-torch.exp(a_log.double()) * torch.nn.functional.softplus(a + dt_bias.double(), threshold=700))
    return dict(row=row, a_log=a_log, dt_bias=dt_bias, q=spread(q) / math.sqrt(D), k=spread(k), v=v.view(T, Hh, V), g=decay, beta=torch.sigmoid(b), n=n)


def _carry(S, c, at, n):
    """The plain recurrence over n tokens from a state."""
    out = []
    for t in range(at, at + n):
        S = c["g"][t].view(-1, 1, 1) * S
        u = c["beta"][t].view(-1, 1) * (c["v"][t] - (S * c["k"][t].unsqueeze(-1)).sum(1))
        S = S + c["k"][t].unsqueeze(-1) * u.unsqueeze(1)
        out.append((S * c["q"][t].unsqueeze(-1)).sum(1))
    return torch.stack(out), S


def _run_delta(c, lens, G, Hh, D, V, state, slots, how):
    from spite_amd.csrc import hipops
    dev, T = "cuda:0", sum(lens)
    row, n = c["row"].to(dev), c["n"] + Hh * V
    cu = torch.tensor(np.concatenate([[0], np.cumsum(lens)]), dtype=torch.int32, device=dev)
    q, k, v = row[:, :G * D], row[:, G * D:2 * G * D], row[:, 2 * G * D:n]
    if how == "chunk":                                   # rows that start on 16 bytes, as the convolution leaves them
        qkv = row[:, :n].contiguous()
        q, k, v = qkv[:, :G * D], qkv[:, G * D:2 * G * D], qkv[:, 2 * G * D:]
    scale, gates = torch.empty(T, 2, G, device=dev), torch.empty(T, 2, Hh, device=dev)
    hipops.delta_gates(q, k, row[:, n:n + Hh], row[:, n + Hh:n + 2 * Hh], c["a_log"].to(dev), c["dt_bias"].to(dev), scale, gates, G, Hh, D,
                       q_scale=D ** -0.5)
    out = torch.full((T, Hh * V), float("nan"), device=dev)
    sl = torch.tensor(slots, dtype=torch.int32, device=dev)
    if how == "chunk":
        arr, nc = hipops.delta_chunks(lens, cu.cpu().numpy())
        scratch = torch.full((hipops.delta_chunk_workspace(nc, G, Hh, D),), 255, dtype=torch.uint8, device=dev)
        hipops.delta_chunk(q, k, v, scale, gates, state, out, torch.from_numpy(arr).to(dev), nc, sl, len(lens), scratch, G, Hh, D, V)
    else:
        hipops.delta_scan(q, k, v, scale, gates, state, out, cu, sl, len(lens), G, Hh, D, V, single=how == "single")
    return out.cpu().double().view(T, Hh, V), scale.cpu().double(), gates.cpu().double()


CHUNK_SIZES = [(1, 2, 32, 16), (2, 4, 64, 48), (1, 3, 96, 72), (2, 2, 128, 136)]


@pytest.mark.gpu
@pytest.mark.parametrize("kind", ["random", "same", "resets"])
@pytest.mark.parametrize("how,dtype,G,Hh,D,V",
                         [("scan", "float32", 2, 4, 12, 10), ("scan", "float32", 1, 1, 1, 1), ("scan", "bfloat16", 3, 3, 70, 21), ("scan", "float32", 1, 2, 200, 36)]
                         + [("chunk", "bfloat16") + s for s in CHUNK_SIZES])
def test_delta_recurrence_kernels(how, dtype, G, Hh, D, V, kind):
    """Two steps of several requests over one state tensor, slots apart, the rows of slots that nobody holds NaN; portions
    around the chunk's length, then single tokens through their own kernel; results and states."""
    slots, n_slots = [5, 0, 3, 2], 7
    state = torch.full((n_slots, Hh, D, V), float("nan"), device="cuda:0")
    for s in slots:
        state[s] = 0.0
    S = [torch.zeros(Hh, D, V, dtype=torch.float64) for _ in slots]
    tol = 2e-5 if kind != "same" else 2e-4
    for step, (lens, way) in enumerate((([33, 1, 70, 32], how), ([1, 1, 1, 1], "single"), ([2, 64, 5, 31], how), ([1, 1, 1, 1], how))):
        c = _delta_case(lens, G, Hh, D, V, dtype, 100 * step + D + V, kind)
        got, scale, gates = _run_delta(c, lens, G, Hh, D, V, state, slots, way)
        at = 0
        assert float((gates[:, 0].exp() - c["g"]).abs().max()) < 1e-6 and float((gates[:, 1] - c["beta"]).abs().max()) < 1e-6
        for i, n in enumerate(lens):
            want, S[i] = _carry(S[i], c, at, n)
            size = float(want.abs().max()) + 1e-3
            assert float((got[at:at + n] - want).abs().max()) < tol * max(size, float(S[i].abs().max()) * 0.3), (step, i)
            at += n
            st = state[slots[i]].cpu().double()
            assert float((st - S[i]).abs().max()) < tol * (float(S[i].abs().max()) + 1e-3), (step, i)
            S[i] = st                                    # (from the engine's state on: one step's error at a time)
    assert bool(torch.isnan(state[[1, 4, 6]]).all())


@pytest.mark.gpu
def test_delta_kernels_agree():
    """Token by token and in chunks: the same numbers to the last bits that fp32 sums leave, far below a bfloat16 step."""
    lens, (G, Hh, D, V) = [200, 3], (2, 4, 128, 64)
    c = _delta_case(lens, G, Hh, D, V, "bfloat16", 5)
    outs = []
    for how in ("scan", "chunk"):
        state = torch.zeros(2, Hh, D, V, device="cuda:0")
        o, _, _ = _run_delta(c, lens, G, Hh, D, V, state, [1, 0], how)
        outs.append((o, state.cpu().double()))
    for x, y in zip(*outs):
        assert float((x - y).abs().max()) < 3e-6 * float(x.abs().max())


@pytest.mark.gpu
def test_delta_kernels_refuse():
    from spite_amd.csrc import hipops
    c = _delta_case([4], 1, 2, 40, 16, "bfloat16", 1)
    state = torch.zeros(1, 2, 40, 16, device="cuda:0")
    with pytest.raises(hipops.KernelError, match="key channels"):
        _run_delta(c, [4], 1, 2, 40, 16, state, [0], "chunk")
    with pytest.raises(hipops.KernelError):
        _run_delta(c, [4], 1, 2, 40, 16, state[:, :1].contiguous(), [0], "scan")
    with pytest.raises(hipops.KernelError):
        _run_delta(c, [4], 1, 2, 40, 16, state, [0], "single")       # four tokens of one entry are no step of single tokens
    big = _delta_case([2], 1, 1, 300, 4, "float32", 1)
    with pytest.raises(hipops.KernelError, match="at most"):
        _run_delta(big, [2], 1, 1, 300, 4, torch.zeros(1, 1, 300, 4, device="cuda:0"), [0], "scan")


@pytest.mark.gpu
@pytest.mark.parametrize("dtype,D,Vd,rot,page,stored", [("float32", 12, 10, 6, 8, 12), ("bfloat16", 64, 32, 20, 32, 64), ("bfloat16", 48, 64, 48, 32, 64),
                                                       ("bfloat16", 10, 6, 2, 16, 10), ("float32", 6, 4, 0, 4, 6)])
def test_turned_and_normed_heads_kernel(dtype, D, Vd, rot, page, stored):
    """Neighbours turn and every head of q and k is divided by its root mean square, in rows of both kernels' kinds."""
    from spite_amd.csrc import hipops
    g = torch.Generator().manual_seed(D)
    dt = getattr(torch, dtype)
    T, HQ, G, eps, base = 9, 4, 2, 1e-3, 500.0
    row = (torch.randn(T, (HQ + G) * D + G * Vd + 3, generator=g) * torch.rand(T, 1, generator=g)).to(dt)
    kp, vp = torch.zeros(4, G, page, stored, dtype=dt, device="cuda:0"), torch.zeros(4, G, Vd, page, dtype=dt, device="cuda:0")
    pos = [0, 1, 2, 3, 4, 5, 6, 7, 8]
    slots = torch.randperm(4 * page, generator=g)[:T].to(torch.int32).cuda()
    q = torch.full((T, HQ * stored), 5.0, dtype=dt, device="cuda:0")
    freq = torch.tensor([base ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=torch.float32).cuda() if rot else None
    hipops.qkv_prepare(row.cuda(), q, kp, vp, torch.tensor(pos, dtype=torch.int32).cuda(), slots, HQ, G, G, D, Vd, page, eps=eps, inv_freq=freq, rot=rot,
                       head_norm=True, adjacent=True, stored_dim=stored)
    x = row.double()
    want = []
    for part, heads in ((x[:, :HQ * D], HQ), (x[:, HQ * D:(HQ + G) * D], G)):
        part = part.reshape(T, heads, D)
        want.append(plain.unit_rms(plain.turn_neighbours(part, {"base": base, "dims": rot}) if rot else part, eps))
    tol = 2e-6 if dtype == "float32" else 2e-2
    got = q.cpu().double().view(T, HQ, stored)
    assert float((got[..., :D] - want[0]).abs().max()) < tol * float(want[0].abs().max()) and bool((got[..., D:] == 0).all())
    for t, s in enumerate(slots.cpu().tolist()):
        k = kp[s // page, :, s % page].cpu().double()
        assert float((k[:, :D] - want[1][t]).abs().max()) < tol * float(want[1].abs().max())
        assert torch.equal(vp[s // page, :, :, s % page].cpu().view(-1), row[t, (HQ + G) * D:(HQ + G) * D + G * Vd])


@pytest.mark.gpu
@pytest.mark.parametrize("dtype,n,spare", [("float32", 30, 5), ("bfloat16", 64, 16), ("bfloat16", 30, 1), ("bfloat16", 1000, 0)])
def test_gate_kernel(dtype, n, spare):
    from spite_amd.csrc import hipops
    g = torch.Generator().manual_seed(n)
    dt = getattr(torch, dtype)
    x, w = torch.randn(7, n, generator=g).to(dt), (torch.randn(7, n + spare, generator=g) * 3).to(dt)
    y = x.cuda()
    hipops.gate_rows(y, w.cuda()[:, spare:], y)
    want = x.double() * torch.sigmoid(w.double()[:, spare:])
    assert float((y.cpu().double() - want).abs().max()) < (1e-6 if dtype == "float32" else 1e-2) * float(want.abs().max())
    with pytest.raises(hipops.KernelError):
        hipops.gate_rows(y, w.cuda()[:, :n - 1], y)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype,heads,V", [("bfloat16", 5, 48), ("bfloat16", 3, 128), ("bfloat16", 2, 256), ("bfloat16", 2, 264), ("bfloat16", 3, 20), ("float32", 3, 48)])
def test_head_norm_and_gate_kernel(dtype, heads, V):
    """Every head on its own, one weight for all, silu of a column range: rows that a lane moves 16 bytes at a time and others."""
    from spite_amd.csrc import hipops
    g = torch.Generator().manual_seed(V)
    dt = getattr(torch, dtype)
    T, n = 7, heads * V
    o, w, z = torch.randn(T, n, generator=g), torch.rand(V, generator=g) + 0.5, (torch.randn(T, n + 16, generator=g) * 2).to(dt)
    y = torch.empty(T, n, dtype=dt, device="cuda:0")
    hipops.gated_group_norm(o.cuda(), w.cuda(), y, V, 1e-3, gate=z.cuda()[:, 16:], act="silu")
    want = plain.norm(o.double().view(T, heads, V), w.double(), 1e-3).view(T, n) * plain.silu(z.double()[:, 16:])
    assert float((y.cpu().double() - want).abs().max()) < (1e-5 if dtype == "float32" else 1e-2) * float(want.abs().max())


@pytest.mark.gpu
@pytest.mark.parametrize("E,top", [(6, 2), (1, 1), (70, 5), (300, 66), (8, 8)])
def test_router_kernel(E, top):
    """The bias is part of the logits: in the choice and in the softmax over the taken."""
    from spite_amd.csrc import hipops
    g = torch.Generator().manual_seed(E + top)
    T = 21
    z, b = torch.randn(T, E, generator=g), torch.randn(E, generator=g) * 2
    expert = torch.empty(T * top, dtype=torch.int32, device="cuda:0")
    weight = torch.empty(T * top, dtype=torch.float32, device="cuda:0")
    hipops.router_topk(z.cuda(), b.cuda(), expert, weight, top, scoring="softmax_taken_biased")
    full = (z + b).double()
    want = torch.sort(full, dim=-1, descending=True, stable=True).indices[:, :top]
    assert torch.equal(expert.cpu().view(T, top).long(), want)
    assert float((weight.cpu().view(T, top).double() - torch.softmax(full.gather(1, want), -1)).abs().max()) < 1e-6


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_query_latent_without_a_cache_row(dtype):
    """A layer that reads another layer's latent norms its queries' latent alone."""
    from spite_amd.csrc import hipops
    g = torch.Generator().manual_seed(4)
    dt = getattr(torch, dtype)
    T, Q, R, Hh = 5, 14, 20, 3
    raw, w = torch.randn(T, Q, generator=g).to(dt), torch.rand(Q, generator=g) + 0.5
    cq = torch.empty(T, Q, dtype=dt, device="cuda:0")
    pages = torch.full((2, 1, 4, R), 3.0, dtype=dt, device="cuda:0")
    rows, offs = torch.empty(Hh * T, dtype=torch.int32, device="cuda:0"), torch.empty(Hh + 1, dtype=torch.int32, device="cuda:0")
    qa = torch.empty(T * Hh, R, dtype=dt, device="cuda:0")
    hipops.latent_prepare(None, None, qa, pages, torch.arange(T, dtype=torch.int32).cuda(), None, None, None, 1e-4, Hh, 10, 0, R, 0, False, rows, offs,
                          query_latent=(raw.cuda(), w.cuda(), cq))
    want = plain.norm(raw.double(), w.double(), 1e-4)
    assert float((cq.cpu().double() - want).abs().max()) < (1e-6 if dtype == "float32" else 1e-2) * float(want.abs().max())
    assert rows.cpu().view(Hh, T).tolist() == [[t * Hh + h for t in range(T)] for h in range(Hh)] and bool((pages == 3.0).all())
    with pytest.raises(hipops.KernelError):
        hipops.latent_prepare(None, None, qa, pages, torch.arange(T, dtype=torch.int32).cuda(), None, None, None, 1e-4, Hh, 10, 0, R, 0, False, rows, offs)


# ------------------------------------------------------------------------------------------ the model in the engine
@pytest.fixture(scope="module")
def models(tmp_path_factory):
    made = {}

    def get(name, dtype):
        if (name, dtype) not in made:
            folder = tmp_path_factory.mktemp(f"porarax_{name}_{dtype}")
            kw = {} if dtype == "float32" else dict(gain=1.5, std=0.05)
            made[(name, dtype)] = (folder, make_model(folder, CONFIGS[name], seed=11 + len(name), dtype=dtype, **kw))
        return made[(name, dtype)]
    return get


@pytest.mark.gpu
@pytest.mark.parametrize("name", ["small", "wide", "ones"])
def test_every_layer_against_plain(models, name):
    """The stream after each layer of a whole prompt, in true 32-bit."""
    from spite_amd.engine.engine import StepEntry, StepMeta
    cfg = CONFIGS[name]
    folder, weights = models(name, "float32")
    toks = H.random_tokens(cfg["vocab"], 37, 3)
    streams = []
    plain.forward(toks, weights, cfg, streams=streams)
    eng = engine(folder, "float32", name)
    slot = eng.admit()
    eng.cache.reserve_all([(slot, len(toks))])
    meta = StepMeta(eng, [StepEntry(slot, toks, [0])])
    eng._step_ws.reset()
    m, state, seen = eng.model, {}, 0
    for u in range(m.n_units()):
        kind, _, i, _ = m._units[u]
        m.run_units(u, u + 1, state, meta.ctx, eng.cache, meta, eng._arenas, eng._step_ws)
        if kind == "stage" and m._units[u + 1][2] != i:
            x = state["h"].clone()
            for p in state["pending"]:
                x += p[:x.shape[0]]
            ref = streams[seen]
            assert float((x.cpu().double() - ref).abs().max()) <= 2e-5 * float(ref.abs().max()), f"layer {seen}"
            seen += 1
    assert seen == len(streams) == len(cfg["layers"])


@pytest.mark.gpu
@pytest.mark.parametrize("name", ["small", "wide", "ones"])
@pytest.mark.parametrize("schedule", ["whole", "tail", "portions", "mixed"])
def test_float32_against_plain(models, name, schedule):
    """True 32-bit: every schedule gives the plain implementation's logits at every position.  Pools start poisoned and
    are small: pages and slots are used again in the mixed schedule."""
    cfg = CONFIGS[name]
    folder, weights = models(name, "float32")
    reqs = requests(cfg["vocab"], LENGTHS[name], 5)
    ref = plain_rows(cfg, weights, reqs)
    steps = {"whole": H.schedule_whole, "tail": lambda r: H.schedule_tail_one_by_one(r, tail=28),
             "portions": H.schedule_portions, "mixed": lambda r: H.schedule_mixed(r, seed=3, max_live=4)}[schedule](reqs)
    eng = engine(folder, "float32", name, cache_tokens=4 * (max(LENGTHS[name]) + PAGE[name]))
    poison(eng)
    got = H.collect(steps, H.run_trace_inprocess(eng, steps), cfg["vocab"])
    err, where = H.max_diff(got, ref)
    assert err <= 2e-4 * scale_of(ref), f"{err} at {where} (scale {scale_of(ref)})"
    assert all(eng.cache.free_pages(g) == eng.cache.total_pages(g) for g in range(eng.cache.n_groups()))


@pytest.mark.gpu
@pytest.mark.parametrize("name", ["small", "wide"])
def test_bfloat16_against_plain_and_itself(models, name):
    """bfloat16 through the serving kernels: whole prompts against the plain implementation with the experts that
    the engine took, then the other schedules against the whole prompts with those experts."""
    cfg = CONFIGS[name]
    folder, weights = models(name, "bfloat16")
    reqs = requests(cfg["vocab"], LENGTHS[name], 8)
    eng = engine(folder, "bfloat16", name, cache_tokens=4 * (max(LENGTHS[name]) + PAGE[name]))
    if name == "wide":
        assert not eng.slow_paths, eng.slow_paths
    poison(eng)
    whole, routing = H.schedule_whole(reqs), {}
    rows = H.collect(whole, H.run_trace_inprocess(eng, whole, routing=routing), cfg["vocab"])
    experts = experts_of(cfg, whole, routing)
    ref = plain_rows(cfg, weights, reqs, taken=experts)
    scale = scale_of(ref)
    close_in_16_bits(rows, ref, scale, 0.06)
    own = {}
    plain_rows(cfg, weights, reqs, chosen=own)
    total = sum(int(e.numel()) for per in experts.values() for e in per)
    same = sum(int((torch.sort(a, 1).values == torch.sort(b, 1).values).sum()) for r in experts for a, b in zip(experts[r], own[r]))
    assert same >= 0.85 * total
    for steps in (H.schedule_tail_one_by_one(reqs, tail=28), H.schedule_portions(reqs), H.schedule_mixed(reqs, seed=4, max_live=4)):
        got = H.collect(steps, H.run_trace_inprocess(eng, steps, take=experts_for(cfg, steps, experts)), cfg["vocab"])
        err, where = H.max_diff(got, rows)
        assert err <= 0.06 * scale, f"{err} at {where} (scale {scale})"


def _one_layer(mixer, mlp=None, width=40, vocab=64):
    return {"architecture": "Porarax", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "layers": [_layer(mixer, mlp)]}


@pytest.mark.gpu
@pytest.mark.parametrize("dtype,wide", [("float32", False), ("bfloat16", True)])
@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("owner_window,reader_window,mute", [(11, None, False), (5, 11, False), (33, 11, True), (None, 11, True)])
def test_window_edges(tmp_path, dtype, wide, decoded, owner_window, reader_window, mute):
    """The logits at i do not move at all when the token just outside the window changes and move when the first one
    inside does: a latent's owner alone; a reader whose window is wider than the owner's; a reader under a narrower
    window than the owner's (whose own result is muted, so that only the reader's window is left).  Prompts and decoding."""
    more = 34 if wide else 0                             # windows that end inside pages and blocks of keys
    edge = (reader_window or owner_window) + more
    size = dict(heads=4, dim=64, vdim=32, kv_rank=64, q_rank=48, scale=0.125) if wide else dict(heads=3, dim=12, vdim=8, kv_rank=18, q_rank=10, scale=0.3)
    cfg = _one_layer(_latent(**size, window=None if owner_window is None else owner_window + more), None, width=128 if wide else 40)
    if reader_window is not None:
        cfg["layers"].append(_layer(_latent(**size, window=edge, kv_from=0), _moe(3, 2, 16, 1.0)))
    t = planted(cfg, 2, gain=1.0)
    if mute:
        t["l0.mix.o"] = torch.zeros_like(t["l0.mix.o"])
    from spite_amd import Engine
    from spite_amd.weights.random_init import write_random_model
    write_random_model(str(tmp_path), cfg, 2, dtype=dtype, overrides=t)
    eng = Engine(str(tmp_path), dtype=dtype, page_size=32 if wide else 8, cache_tokens=512, max_requests=2, device="cuda:0")
    n = 3 * edge + 9
    base = H.random_tokens(64, n, 1)

    def run(at):
        toks = list(base)
        if at is not None:
            toks[at] = (base[at] + 7) % 64
        reqs = {"a": toks}
        steps = H.schedule_tail_one_by_one(reqs, tail=n - edge - 3) if decoded else H.schedule_whole(reqs)
        return H.collect(steps, H.run_trace_inprocess(eng, steps), 64)
    ref = run(None)
    for i in (edge + 4, 2 * edge + 1, n - 1):
        top = float(np.abs(ref[("a", i)]).max())
        for out in (i - edge, 0, (i - edge) // 2):
            assert np.array_equal(run(out)[("a", i)], ref[("a", i)]), f"position {i} sees the token at {out}"
        for inside in (i - edge + 1, i - 1):
            assert float(np.abs(run(inside)[("a", i)] - ref[("a", i)]).max()) > 1e-4 * top, f"position {i} misses the token at {inside}"


def _far_tokens(n, key_tok, query_tok, at, queries, seed=9):
    toks = [x if x not in (key_tok, query_tok) else 11 for x in H.random_tokens(64, n, seed)]
    toks[at] = key_tok
    for i in queries:
        toks[i] = query_tok
    return toks


def _against_plain(folder, cfg, toks, at, queries, dtype, page, least, tail):
    weights = H.read_weights(str(folder))
    without = list(toks)
    without[at] = 11
    ref, other = plain.forward(toks, weights, cfg), plain.forward(without, weights, cfg)
    scale = float(ref.abs().max())
    far = float((ref[queries] - other[queries]).abs().amax(1).min())
    assert far > least * scale, far / scale               # the plain implementation depends on the far token
    from spite_amd import Engine
    eng = Engine(str(folder), dtype=dtype, page_size=page, cache_tokens=512, max_requests=2, device="cuda:0")
    poison(eng)
    for steps in (H.schedule_tail_one_by_one({"a": toks}, tail=tail), H.schedule_portions({"a": toks}, sizes=(64, 2, 45, 30))):
        got = H.collect(steps, H.run_trace_inprocess(eng, steps), 64)
        rows = {("a", i): ref[i].float().numpy() for i in range(len(toks))}
        err, where = H.max_diff(got, rows)
        assert err <= (2e-4 if dtype == "float32" else 0.06) * scale, f"{err} at {where} (scale {scale})"


@pytest.mark.gpu
@pytest.mark.parametrize("kind", ["attention", "latent", "reader"])
@pytest.mark.parametrize("dtype,wide", [("float32", False), ("bfloat16", True)])
def test_one_far_key_stands_out(tmp_path, dtype, wide, kind):
    """One token stands at position 3 only; another stands hundreds of keys later, in the prompt and among 130 decoded
    tokens, and its query scores the far key far above all others: through normed heads, through the latents, and through
    another layer's latent."""
    key_tok, query_tok, queries = 7, 9, [150, 280, 320]
    if kind == "attention":
        mixer = _attention(4, 2, 64, 32, 0.22, 1000.0, 16) if wide else _attention(3, 3, 12, 10, 1.5, 1000.0, 4)
        cfg, name = _one_layer(mixer, None, width=128 if wide else 40), "l0"
    else:
        size = dict(heads=4, dim=64, vdim=32, kv_rank=64, q_rank=32, scale=0.125) if wide else dict(heads=3, dim=10, vdim=8, kv_rank=20, q_rank=20, scale=0.3)
        cfg, name = _one_layer(_latent(**size), None, width=128 if wide else 40), "l0"
        if kind == "reader":
            cfg["layers"].append(_layer(_latent(**size, kv_from=0), None))
            name = "l1"
    t = planted(cfg, 3, gain=0.5)
    mx = cfg["layers"][0]["mixer"]
    Hh, D = mx["heads"], mx["dim"]

    def normed(tok, layer):
        h = plain.norm(t["embed"][tok].double(), t[layer + ".norm1"].double(), cfg["norm"]["eps"])
        return (h / h.norm()).float()
    hk, hq = normed(key_tok, "l0"), normed(query_tok, name)
    if kind == "attention":
        for h in range(Hh):
            t["l0.mix.q"][h * D + D - 1] = 1.5 * hq
        for g in range(mx["kv_heads"]):
            t["l0.mix.k"][g * D + D - 1] = 1.5 * hk
    else:
        if kind == "reader":
            t["l0.mix.o"] = torch.zeros_like(t["l0.mix.o"])
        t[name + ".mix.dq"], t["l0.mix.dkv"] = t[name + ".mix.dq"] * 4.0, t["l0.mix.dkv"] * 4.0
        t[name + ".mix.dq"][0], t["l0.mix.dkv"][0] = 2.0 * hq, 2.0 * hk
        for h in range(Hh):
            at = h * D + D - 1
            t[name + ".mix.uq"][at], t[name + ".mix.uk"][at] = 0.0, 0.0
            t[name + ".mix.uq"][at, 0], t[name + ".mix.uk"][at, 0] = 2.2, 2.2
        t[name + ".mix.uv"] = t[name + ".mix.uv"] * 3.0
    t[name + ".mix.o"] = t[name + ".mix.o"] * 8.0
    from spite_amd.weights.random_init import write_random_model
    write_random_model(str(tmp_path), cfg, 3, dtype=dtype, overrides=t)
    toks = _far_tokens(330, key_tok, query_tok, 3, queries)
    _against_plain(tmp_path, cfg, toks, 3, queries, dtype, 32 if wide else 8, 0.05 if dtype == "float32" else 0.1, 130)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype,wide", [("float32", False), ("bfloat16", True)])
def test_far_token_in_the_state(tmp_path, dtype, wide):
    """One token is written with a step size near 1 while all others write next to nothing and nothing decays: hundreds of
    tokens later, prompts and decoding, the state still holds it."""
    key_tok, query_tok, queries = 7, 9, [150, 330, 400]
    cfg = _one_layer(_delta(4, 2, 64, 32, 2) if wide else _delta(3, 3, 12, 10, 3), None, width=128 if wide else 40)
    t = planted(cfg, 5)
    t["embed"][:, 0] = 2.0                                # a direction that all tokens share: a bias for the step size
    mx = cfg["layers"][0]["mixer"]
    h = plain.norm(t["embed"].double(), t["l0.norm1"].double(), cfg["norm"]["eps"])
    own = h[key_tok].clone()
    own[0] = 0.0
    own = (own / own.dot(h[key_tok])).float()
    shared = torch.zeros_like(own)
    shared[0] = 1.0 / float(h[:, 0].mean())
    for head in range(mx["heads"]):
        t["l0.mix.b"][head] = 10.0 * own - 7.0 * shared
    t["l0.mix.A_log"][:] = -9.0
    t["l0.mix.o"] = t["l0.mix.o"] * 3.0
    from spite_amd.weights.random_init import write_random_model
    write_random_model(str(tmp_path), cfg, 5, dtype=dtype, overrides=t)
    toks = _far_tokens(420, key_tok, query_tok, 3, queries)
    _against_plain(tmp_path, cfg, toks, 3, queries, dtype, 32 if wide else 8, 0.02, 130)


@pytest.mark.gpu
@pytest.mark.parametrize("name,dtype", [("small", "float32"), ("wide", "bfloat16")])
def test_slots_and_pages_are_used_again(models, name, dtype):
    """Requests that take one slot and its pages one after another read nothing of each other: the first one's logits
    come back bit by bit after another request has been there."""
    cfg = CONFIGS[name]
    folder, _ = models(name, dtype)
    eng = engine(folder, dtype, name, max_requests=1, cache_tokens=96)
    a, b = H.random_tokens(cfg["vocab"], 60, 1), H.random_tokens(cfg["vocab"], 75, 2)
    outs = []
    for toks in (a, b, a):
        free = [eng.cache.free_pages(g) for g in range(eng.cache.n_groups())]
        steps = H.schedule_portions({"x": toks}, sizes=(1, 2, 33, 3))
        outs.append(H.collect(steps, H.run_trace_inprocess(eng, steps), cfg["vocab"]))
        assert [eng.cache.free_pages(g) for g in range(eng.cache.n_groups())] == free
        for g in eng.cache.groups:
            for half in g.halves():
                if half.numel():
                    half.fill_(float("nan"))
    for k in outs[0]:
        assert np.array_equal(outs[0][k], outs[2][k]) and np.isfinite(outs[1][("x", 74)]).all()


@pytest.mark.gpu
@pytest.mark.parametrize("name", ["small", "wide"])
def test_greedy_generation(models, name):
    """Through the engine's own entry point and scheduler: prompts of unequal length, more new tokens than the
    windows are long, in true 32-bit: the plain implementation's greedy tokens."""
    cfg = CONFIGS[name]
    folder, weights = models(name, "float32")
    prompts = [H.random_tokens(cfg["vocab"], n, 40 + n) for n in (1, 19, 7)]
    eng = engine(folder, "float32", name, cache_tokens=512, max_batch_tokens=16)
    n_new = 30 if name == "small" else 10
    got = eng.generate(prompts, max_tokens=n_new, temperature=0.0)
    compared = 0
    for p, g in zip(prompts, got):
        toks = list(p)
        for k in range(n_new):
            last = plain.forward(toks, weights, cfg)[-1]
            top = torch.topk(last, 2).values
            if float(top[0] - top[1]) < 1e-3 * float(last.abs().max()):
                break                                              # a tie at 32-bit precision: what follows may differ
            assert g[k] == int(torch.argmax(last)), f"token {k} of a prompt of {len(p)}"
            toks.append(g[k])
            compared += 1
    assert compared >= n_new


@pytest.mark.gpu
def test_decode_steps_replay_graphs(models):
    """Decode steps of one shape are captured and replayed; every replay gives the eager logits (recurrent
    states and the convolution's inputs move on inside the graph)."""
    cfg = CONFIGS["wide"]
    folder, _ = models("wide", "bfloat16")
    reqs = requests(cfg["vocab"], [40, 41], 21)
    steps = [{"step": 0, "entries": [{"id": r, "tokens": t[:20], "want": [19]} for r, t in reqs.items()], "end": []}]
    steps += [{"step": 1 + i, "entries": [{"id": r, "tokens": [t[20 + i]], "want": [0]} for r, t in reqs.items()], "end": []} for i in range(20)]
    outs = []
    for graphs in (False, True):
        eng = engine(folder, "bfloat16", "wide", graphs=graphs)
        outs.append(H.run_trace_inprocess(eng, copy.deepcopy(steps)))
        assert (eng.graph_replays > 10) == graphs
    for k in outs[0]:
        assert np.array_equal(outs[0][k], outs[1][k]), f"step {k}"


def random_config(seed, aligned=False):
    """A configuration drawn from a seed: layer count and order, heads, sizes, windows, readers and constants all vary; now
    and then a value is 1 or sizes are odd.  ``aligned``: sizes that the bfloat16 runs take on the matrix units in one
    kernel or another."""
    rng = np.random.RandomState(seed)
    pick = lambda *xs: xs[rng.randint(len(xs))]
    ff = lambda: int(pick(32, 64, 96)) if aligned else int(pick(1, 4, 12, 20))
    layers, owners = [], {}
    for i in range(int(pick(1, 2, 4, 6))):
        experts = int(pick(1, 2, 5, 8))
        mlp = pick(None, *[_moe(experts, int(rng.randint(min(experts, 4))) + 1, ff(), float(pick(0.3, 0.8, 1.5, 7.0)))] * 3)
        kind = pick("latent", "latent", "attention", "delta")
        if kind == "attention":
            kv, dim = int(pick(1, 2, 3)), int(pick(32, 64, 128)) if aligned else int(pick(1, 2, 7, 12, 20))
            dims = min(int(pick(0, 2, 16, 32, 128)) if aligned else int(pick(0, 2, 6, 12)), dim // 2 * 2)
            mixer = _attention(kv * int(pick(1, 2, 4)), kv, dim, int(pick(32, 64, 128)) if aligned else int(pick(1, 5, 12)), float(pick(0.1, 0.25, 0.5)),
                               float(pick(100.0, 10000.0)), dims)
        elif kind == "latent":
            owner = pick(None, *owners) if owners else None
            rank = owners[owner] if owner is not None else (int(pick(32, 64, 200)) if aligned else int(pick(1, 7, 18)))
            mixer = _latent(int(pick(1, 3, 8)), int(pick(32, 64)) if aligned else int(pick(1, 6, 12)), int(pick(32, 48)) if aligned else int(pick(1, 5, 9)),
                            rank, int(pick(32, 64, 96)) if aligned else int(pick(1, 5, 33)), float(pick(0.1, 0.25)), window=pick(None, 1, 2, 7, 24, 33, 64),
                            kv_from=owner)
            if owner is None:
                owners[i] = rank
        else:
            kv = int(pick(1, 2, 3))
            mixer = _delta(kv * int(pick(1, 2, 4)), kv, int(pick(32, 64, 96, 128)) if aligned else int(pick(1, 2, 7, 12, 20)),
                           int(pick(16, 40, 64, 128)) if aligned else int(pick(1, 4, 5, 12)), int(pick(1, 2, 3, 4, 6)))
        layers.append(_layer(mixer, mlp))
    return {"architecture": "Porarax", "vocab": int(pick(50, 128, 257)), "width": int(pick(64, 128, 256)) if aligned else int(pick(24, 37, 48, 64)),
            "norm": {"eps": float(pick(1e-6, 1e-5, 1e-3))}, "layers": layers}


@pytest.mark.gpu
@pytest.mark.parametrize("seed", list(range(8)) + list(range(100, 108)))
def test_random_configurations(tmp_path, seed):
    """Whatever the configuration says: true 32-bit against the plain implementation, whole prompts and a mixed
    schedule through small pages; then bfloat16 against itself across schedules and, loosely, against the plain
    implementation."""
    cfg = random_config(seed, aligned=seed >= 100)
    rng = np.random.RandomState(seed + 100)
    page = int(rng.choice([4, 16, 32, 64]))
    weights = make_model(tmp_path / "f32", cfg, seed=seed, dtype="float32", gain=2.0)
    reqs = requests(cfg["vocab"], [41, 1, 70, 2, 19], seed)
    ref = plain_rows(cfg, weights, reqs)
    from spite_amd import Engine
    eng = Engine(str(tmp_path / "f32"), dtype="float32", page_size=page, cache_tokens=4 * (70 + page), max_requests=4, device="cuda:0")
    poison(eng)
    for steps in (H.schedule_whole(reqs), H.schedule_mixed(reqs, seed=seed, max_live=4)):
        got = H.collect(steps, H.run_trace_inprocess(eng, steps), cfg["vocab"])
        err, where = H.max_diff(got, ref)
        assert err <= 3e-4 * scale_of(ref), f"{err} at {where} (scale {scale_of(ref)}): {cfg}"
    del eng
    weights = make_model(tmp_path / "bf16", cfg, seed=seed, dtype="bfloat16", gain=1.5, std=0.05)
    eng = Engine(str(tmp_path / "bf16"), dtype="bfloat16", page_size=page, cache_tokens=4 * (70 + page), max_requests=4, device="cuda:0")
    poison(eng)
    whole, routing = H.schedule_whole(reqs), {}
    rows = H.collect(whole, H.run_trace_inprocess(eng, whole, routing=routing), cfg["vocab"])
    experts = experts_of(cfg, whole, routing) if tops(cfg) else None
    ref = plain_rows(cfg, weights, reqs, taken=experts)
    scale = scale_of(ref)
    close_in_16_bits(rows, ref, scale, 0.08)
    steps = H.schedule_mixed(reqs, seed=seed + 1, max_live=4)
    got = H.collect(steps, H.run_trace_inprocess(eng, steps, take=experts_for(cfg, steps, experts) if experts else None), cfg["vocab"])
    err, where = H.max_diff(got, rows)
    assert err <= 0.08 * scale, f"{err} at {where} (scale {scale}): {cfg}"


@pytest.mark.gpu
def test_replay_program(models):
    """The replay program on a model folder, as a child process: a mixed schedule in true 32-bit gives the plain
    implementation's logits."""
    cfg = CONFIGS["small"]
    folder, weights = models("small", "float32")
    reqs = requests(cfg["vocab"], [30, 1, 47, 12, 22], 77)
    steps = H.schedule_mixed(reqs, seed=9, max_live=4)
    out = H.run_trace_program(str(folder), "float32", steps, max_tokens=4 * 64, extra=["--page-size", "16", "--max-requests", "4"])
    got = H.collect(steps, out, cfg["vocab"])
    ref = plain_rows(cfg, weights, reqs)
    err, where = H.max_diff(got, ref)
    assert err <= 2e-4 * scale_of(ref), f"{err} at {where}"


@pytest.mark.gpu
def test_command_line_and_sampling(models):
    """`spite run` on the model's folder: the greedy tokens of `Engine.generate`; and sampling with a seed through the
    framework's sampler gives the same tokens twice and other tokens than greedy somewhere."""
    cfg = CONFIGS["small"]
    folder, _ = models("small", "float32")
    p = H.random_tokens(cfg["vocab"], 9, 21)
    eng = engine(folder, "float32", "small", cache_tokens=256)
    want = eng.generate([p], max_tokens=12, temperature=0.0)[0]
    out = subprocess.run([sys.executable, os.path.join(H.ROOT, "bin", "spite"), "run", "-m", str(folder), "--prompt-ids",
                          ",".join(map(str, p)), "--max-tokens", "12", "--temperature", "0", "--dtype", "fp32",
                          "--ctx", "64", "--page-size", "16"], capture_output=True, text=True, timeout=120)
    assert out.returncode == 0, out.stderr
    assert out.stdout.strip().splitlines()[-1].split() == [str(t) for t in want]
    a = eng.generate([p, p[:4]], max_tokens=12, temperature=12.0, seed=5)
    b = eng.generate([p, p[:4]], max_tokens=12, temperature=12.0, seed=5)
    assert a == b and a[0] != want
