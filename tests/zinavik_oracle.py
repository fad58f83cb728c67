"""Plain, slow float64 implementation of the Zinavik decoder, one function per mechanism,
written from the design's equations. It reads a config DICT (the layout of a model folder's
config.json) and a dict of named tensors, and shares no code with hipserve: the tests
compare the engine against it.

Notation: xs [streams, n, width] are one sequence's residual streams, positions count from 0.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def rms_unit(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def lin(w, x):
    """Weights are stored [out, in]; rows of x are tokens."""
    return x @ w.T


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


# ---------------------------------------------------------------- rotation
def yarn_frequencies(rot):
    """(angle per position of every rotated pair, factor on cos and sin)."""
    dims, base, sc = rot["dims"], rot["base"], rot.get("scaling")
    freqs = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not sc:
        return torch.tensor(freqs, dtype=F64), 1.0

    def dim_of(turns):   # the (real-valued) pair index whose wavelength fits `turns` times into the original length
        return dims * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(dim_of(sc["fast"])), 0)
    hi = min(math.ceil(dim_of(sc["slow"])), dims - 1)
    out = []
    for i, f in enumerate(freqs):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / sc["factor"] * r + f * (1.0 - r))
    return torch.tensor(out, dtype=F64), 0.1 * math.log(sc["factor"]) + 1.0


def rotate_pairs(x, pos, rot):
    """x [n, heads, d]: coordinates (2i, 2i+1), i < dims/2, turn by pos * f_i and grow by the factor."""
    f, amp = yarn_frequencies(rot)
    dims = rot["dims"]
    ang = pos.to(F64)[:, None] * f                                   # [n, dims/2]
    c, s = (torch.cos(ang) * amp)[:, None, :], (torch.sin(ang) * amp)[:, None, :]
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


# ---------------------------------------------------------------- mixers
def window_attention(h, w, m, eps):
    """Left half: w holds q, k, v, g, o."""
    n = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(n)
    q = rms_unit(rotate_pairs(lin(w["q"], h).view(n, H, d), pos, m["rot"]), eps)
    k = rms_unit(rotate_pairs(lin(w["k"], h).view(n, G, d), pos, m["rot"]), eps)
    v = lin(w["v"], h).view(n, G, dv)
    k, v = k.repeat_interleave(H // G, 1), v.repeat_interleave(H // G, 1)
    sc = torch.einsum("ihd,jhd->hij", q, k) * m["scale"]
    i, j = pos[:, None], pos[None, :]
    seen = (j <= i) & ((i - j < m["mask"]["size"]) | (j < m["mask"]["keep_first"]))
    p = torch.softmax(sc.masked_fill(~seen, -math.inf), -1)
    o = torch.einsum("hij,jhv->ihv", p, v).reshape(n, H * dv)
    return lin(w["o"], o * sigmoid(lin(w["g"], h)))


def lightning(h, w, m, eps, state=None):
    """Right half: S <- decay S + k v^T per head, read by q; ``state`` [heads, dim, vdim] carries on."""
    n = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]

    def silu(z):
        return z * sigmoid(z)

    q, k = silu(lin(w["q"], h)).view(n, H, d), silu(lin(w["k"], h)).view(n, H, d)
    v = silu(lin(w["v"], h)).view(n, H, dv)
    lam = torch.tensor(m["decay"], dtype=F64)[:, None, None]
    S = torch.zeros(H, d, dv, dtype=F64) if state is None else state.clone()
    o = torch.empty(n, H, dv, dtype=F64)
    for t in range(n):
        S = lam * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = torch.einsum("hdv,hd->hv", S, q[t])
    o = rms_unit(o.reshape(n, H * dv), eps) * w["norm"] * sigmoid(lin(w["g"], h))
    return lin(w["o"], o), S


def parallel_mixer(h, w, m, eps, state=None):
    left = window_attention(h, sub(w, "left."), m["left"], eps)
    right, S = lightning(h, sub(w, "right."), m["right"], eps, state)
    return m["left_scale"] * left + m["right_scale"] * right, S


# ---------------------------------------------------------------- feed-forward
def clamped_expert(h, gate, up, down, limit):
    g = torch.clamp(lin(gate, h), max=limit)
    u = torch.clamp(lin(up, h), min=-limit, max=limit)
    return lin(down, g * sigmoid(1.702 * g) * (u + 1.0))


def route(h, w, r):
    """Chosen experts [n, top] and their scores [n, top]."""
    s = sigmoid(lin(w["router"], h))
    ids = torch.topk(s, r["top"], dim=-1).indices
    return ids, s.gather(1, ids)


def moe_ff(h, w, f):
    ids, ws = route(h, w, f["router"])
    out = torch.zeros(h.shape[0], w["e0.down"].shape[0], dtype=F64)
    for t in range(h.shape[0]):
        for e, wt in zip(ids[t].tolist(), ws[t]):
            out[t] += clamped_expert(wt * h[t:t + 1], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], f["expert"]["limit"])[0]
    if f.get("shared"):
        y = clamped_expert(h, w["shared.gate"], w["shared.up"], w["shared.down"], f["shared"]["limit"])
        out = out + sigmoid(lin(w["shared.sg"], h)) * y
    return out


# ---------------------------------------------------------------- residual streams
def streams_in(xs, w):
    """The sublayer's input before its norm: sum_s in[s] x_s."""
    return torch.einsum("s,snd->nd", w["in"], xs)


def streams_update(xs, w, y):
    """x_t <- sum_s mix[s, t] x_s + out[t] y, all from the old streams."""
    return torch.einsum("st,snd->tnd", w["mix"], xs) + w["out"][:, None, None] * y


# ---------------------------------------------------------------- the model
def sub(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def layer_runs(cfg):
    """Layer indices in execution order."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return list(range(n))
    return list(range(lp["start"])) + list(range(lp["start"], lp["stop"])) * lp["times"] + list(range(lp["stop"], n))


def forward(cfg: dict, tensors: dict, tokens, return_layers: bool = False):
    """Logits [n, vocab] of one sequence from position 0; with ``return_layers`` also the sum of the streams after
    every layer run and the recurrent states."""
    W = {k: v.to(F64) for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    xs = x[None].repeat(cfg["streams"], 1, 1)
    after, states = [], []
    for i in layer_runs(cfg):
        L, p = cfg["layers"][i], f"l{i}."
        assert L["type"] == "parallel"
        hc = sub(W, p + "hc1.")
        y, S = parallel_mixer(rms_unit(streams_in(xs, hc), eps) * W[p + "norm1"], sub(W, p + "mix."), L["mixer"], eps)
        states.append(S)
        xs = streams_update(xs, hc, y)
        if L.get("mlp") is not None:
            hc = sub(W, p + "hc2.")
            y = moe_ff(rms_unit(streams_in(xs, hc), eps) * W[p + "norm2"], sub(W, p + "mlp."), L["mlp"])
            xs = streams_update(xs, hc, y)
        after.append(xs.sum(0))
    logits = lin(W["embed"], rms_unit(xs.sum(0), eps) * W["final.norm"])
    if return_layers:
        return logits, torch.stack(after) if after else xs[:0], states
    return logits


# ------------------------------------------------------------------ small configs and random weights
def attn_half(heads=6, kv_heads=2, dim=10, vdim=7, scale=0.4, size=11, keep_first=3, dims=6, base=800.0, factor=3.0,
              original=40, fast=4.0, slow=0.5, scaled=True):
    rot = {"base": base, "dims": dims}
    if scaled:
        rot["scaling"] = {"factor": factor, "original": original, "fast": fast, "slow": slow}
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
            "mask": {"size": size, "keep_first": keep_first}, "rot": rot}


def lightning_half(heads=3, dim=5, vdim=8, decay=None):
    if decay is None:
        decay = [1.0 - 2.0 ** (-1.5 * (h + 1)) for h in range(heads)]
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}


def moe(experts=5, top=2, ff=12, limit=1.5, shared=18, shared_limit=0.9):
    f = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    if shared:
        f["shared"] = {"ff": shared, "limit": shared_limit}
    return f


def layer(left=None, right=None, left_scale=0.7, right_scale=1.3, mlp=None):
    return {"type": "parallel", "mlp": mlp,
            "mixer": {"left": left or attn_half(), "right": right or lightning_half(), "left_scale": left_scale,
                      "right_scale": right_scale}}


def make_config(layers, width=28, vocab=90, eps=1e-5, scale=3.0, streams=3, loop=None):
    cfg = {"architecture": "Zinavik", "embedding": {"scale": scale}, "layers": layers, "norm": {"eps": eps},
           "streams": streams, "vocab": vocab, "width": width}
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def make_weights(cfg, seed=0, gain=1.0):
    """Random checkpoint tensors (values representable in bf16) under the design's names."""
    g = torch.Generator().manual_seed(seed)
    Wd, V, S = cfg["width"], cfg["vocab"], cfg["streams"]

    def rnd(*shape, std=1.0):
        return torch.randn(*shape, generator=g) * std

    def mat(o, i):
        return rnd(o, i, std=gain / math.sqrt(i))

    W = {"embed": rnd(V, Wd, std=1.0 / cfg["embedding"]["scale"]), "final.norm": 1 + rnd(Wd, std=0.2)}
    for i, l in enumerate(cfg["layers"]):
        m, f = l["mixer"], l["mlp"]
        a, r, p = m["left"], m["right"], f"l{i}.mix."
        qs, ks, vs, out = a["heads"] * a["dim"], a["kv_heads"] * a["dim"], a["kv_heads"] * a["vdim"], a["heads"] * a["vdim"]
        W.update({p + "left.q": mat(qs, Wd) * 2, p + "left.k": mat(ks, Wd) * 2, p + "left.v": mat(vs, Wd) * 2,
                  p + "left.g": mat(out, Wd) * 2, p + "left.o": mat(Wd, out)})
        qk, out = r["heads"] * r["dim"], r["heads"] * r["vdim"]
        W.update({p + "right.q": mat(qk, Wd) * 2, p + "right.k": mat(qk, Wd) * 2, p + "right.v": mat(out, Wd) * 2,
                  p + "right.g": mat(out, Wd) * 2, p + "right.o": mat(Wd, out), p + "right.norm": 1 + rnd(out, std=0.2)})
        for q in (1, 2) if f is not None else (1,):
            h = f"l{i}.hc{q}."
            W[f"l{i}.norm{q}"] = 1 + rnd(Wd, std=0.2)
            W[h + "in"] = 1.0 / S + rnd(S, std=0.4)
            W[h + "out"] = 1.0 + rnd(S, std=0.4)
            W[h + "mix"] = 0.8 * torch.eye(S) + rnd(S, S, std=0.3 / math.sqrt(S))
        if f is None:
            continue
        p, n = f"l{i}.mlp.", f["router"]["experts"]
        W[p + "router"] = mat(n, Wd) * 2
        for e in [f"e{e}." for e in range(n)] + (["shared."] if f.get("shared") else []):
            ff = f["shared"]["ff"] if e == "shared." else f["expert"]["ff"]
            W[p + e + "gate"], W[p + e + "up"], W[p + e + "down"] = mat(ff, Wd) * 2, mat(ff, Wd) * 2, mat(Wd, ff)
        if f.get("shared"):
            W[p + "shared.sg"] = mat(1, Wd) * 2
    return {k: v.bfloat16().float() for k, v in W.items()}


def save_checkpoint(path, cfg, W):
    import json
    import os

    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.bfloat16().contiguous() for k, v in W.items()}, os.path.join(path, "model.safetensors"))
    return path
