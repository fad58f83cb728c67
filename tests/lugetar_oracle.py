"""Plain, slow float64 implementation of the Lugetar decoder, one function per mechanism, whole
sequences, token by token where the design is recurrent: no cache, no batching and no code shared
with ``hipserve``. It is what ``tests/test_lugetar.py`` compares the framework with.

A model is (config dict as in ``config.json``, dict of tensors under the checkpoint's names).
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def lin(w, x):
    return x @ w.t()


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return torch.where(x > 30, x, torch.log1p(torch.exp(torch.clamp(x, max=30.0))))


def rms_unit(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def length_unit(x):
    """x / sqrt(sum(x^2) + 1e-6) over the last axis."""
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


# ---------------------------------------------------------------- attention
def frequencies(rot):
    """Angle per position of every pair: base^(-2i/dims); with ``scaling`` long waves are slowed down by ``factor``,
    short ones kept, with a linear blend (in turns over the original length) between ``low`` and ``high``."""
    dims, sc, out = rot["dims"], rot.get("scaling"), []
    for i in range(dims // 2):
        f = rot["base"] ** (-2.0 * i / dims)
        if sc:
            wave = 2.0 * math.pi / f
            if wave > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif wave >= sc["original"] / sc["high"]:
                s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return torch.tensor(out, dtype=F64)


def rotate(x, rot):
    """x [n, heads, dim]: dimension i turns with i + dims / 2 by position * frequency i; the rest is left alone."""
    if not rot or not rot.get("dims"):
        return x
    half = rot["dims"] // 2
    a = torch.arange(x.shape[0], dtype=F64)[:, None] * frequencies(rot)[None]
    c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], -1)


def temperature(n, qt):
    """Query factor of every position: 1 + coef ln(floor((p + 1) / every) + 1)."""
    return torch.tensor([1.0 + qt["coef"] * math.log(math.floor((p + 1) / qt["every"]) + 1.0) for p in range(n)], dtype=F64)


def visible(n, chunk):
    """[query, key]: keys up to the query's position, inside its chunk when there are chunks."""
    i = torch.arange(n)
    ok = i[None] <= i[:, None]
    return ok & (i[:, None] // chunk == i[None] // chunk) if chunk else ok


def attend(q, k, v, scale, ok):
    """q [n, H, d], k [n, G, d], v [n, G, dv]: softmax attention, query head h on key / value head h // (H / G)."""
    n, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(n, H, v.shape[-1], dtype=F64)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].t() * scale).masked_fill(~ok, float("-inf"))
        out[:, h] = torch.softmax(s, -1) @ v[:, g]
    return out


def attention(h, w, m, eps):
    """Grouped-query attention with q / k norms over the whole projection; optional rotation, chunks, temperature."""
    n, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_unit(lin(w["q"], h), eps) * w["q.norm"]
    k = rms_unit(lin(w["k"], h), eps) * w["k.norm"]
    v = lin(w["v"], h)
    q, k = rotate(q.view(n, H, d), m.get("rot")), rotate(k.view(n, G, d), m.get("rot"))
    if m.get("q_temp"):
        q = q * temperature(n, m["q_temp"])[:, None, None]
    o = attend(q, k, v.view(n, G, dv), m["scale"], visible(n, (m.get("mask") or {}).get("size")))
    return lin(w["o"], o.reshape(n, H * dv))


# ---------------------------------------------------------------- gated delta rule with a decay per key channel
def causal_conv(x, w):
    """x [n, C], w [C, taps] (last column: the current token), zeros before the start."""
    n, taps = x.shape[0], w.shape[1]
    xp = torch.cat([torch.zeros(taps - 1, x.shape[1], dtype=F64), x])
    return sum(xp[j:j + n] * w[:, j] for j in range(taps))


def decays(h, w, m):
    """exp(-exp(A_log) softplus(.)) of the bottleneck, [n, heads, dim]."""
    pre = lin(w["a2"], lin(w["a1"], h)) + w["dt_bias"]
    return torch.exp(-torch.exp(w["A_log"])[None, :, None] * softplus(pre).view(h.shape[0], m["heads"], m["dim"]))


def delta_scan(q, k, v, beta, g):
    """Per head: S <- g S (rows); u = beta (v - S^T k); S <- S + k u^T; o = S^T q. q, k [n, heads, dim]."""
    n, H, dv = v.shape
    o = torch.zeros(n, H, dv, dtype=F64)
    S = torch.zeros(H, q.shape[-1], dv, dtype=F64)
    for h in range(H):
        for t in range(n):
            S[h] = g[t, h][:, None] * S[h]
            u = beta[t, h] * (v[t, h] - S[h].t() @ k[t, h])
            S[h] = S[h] + torch.outer(k[t, h], u)
            o[t, h] = S[h].t() @ q[t, h]
    return o, S


def channel_delta(h, w, m, eps, return_state=False):
    n, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = silu(causal_conv(lin(w["q"], h), w["q.conv"])).view(n, G, d)
    k = silu(causal_conv(lin(w["k"], h), w["k.conv"])).view(n, G, d)
    v = silu(causal_conv(lin(w["v"], h), w["v.conv"])).view(n, H, dv)
    q, k = length_unit(q) * d ** -0.5, length_unit(k)
    q, k = q.repeat_interleave(H // G, 1), k.repeat_interleave(H // G, 1)
    o, S = delta_scan(q, k, v, sigmoid(lin(w["b"], h)), decays(h, w, m))
    gate = sigmoid(lin(w["g2"], lin(w["g1"], h))).view(n, H, dv)
    y = lin(w["o"], (rms_unit(o, eps) * w["norm"] * gate).reshape(n, H * dv))
    return (y, S) if return_state else y


def parallel_mixer(h, w, m, eps):
    """Half the sum of the two halves' outputs, each normed over the width with a weight of its own."""
    a = attention(h, sub(w, "left."), m["left"], eps)
    b = channel_delta(h, sub(w, "right."), m["right"], eps)
    return 0.5 * (rms_unit(a, eps) * w["left.out"] + rms_unit(b, eps) * w["right.out"])


# ---------------------------------------------------------------- feed-forwards
def clamped_ff(h, w, limit):
    g = torch.clamp(lin(w["gate"], h), max=limit)
    u = torch.clamp(lin(w["up"], h), -limit, limit)
    return lin(w["down"], g * sigmoid(1.702 * g) * (u + 1.0))


def expert(h, w):
    return lin(w["down"], silu(lin(w["gate"], h)) * lin(w["up"], h))


def route(h, w, r):
    """Ids and weights [n, top]: the largest sigmoid scores among the experts of the best groups."""
    s = sigmoid(lin(w["router"], h))
    n, E = s.shape
    groups = r.get("groups") or {"count": 1, "keep": 1}
    count, keep = groups["count"], groups["keep"]
    per, ids = E // count, []
    for t in range(n):
        of = [sum(sorted(s[t, g * per:(g + 1) * per].tolist())[-2:]) for g in range(count)]
        kept = sorted(range(count), key=lambda g: (-of[g], g))[:keep]
        cand = [e for e in range(E) if e // per in kept]
        ids.append(sorted(cand, key=lambda e: (-float(s[t, e]), e))[:r["top"]])
    ids = torch.tensor(ids)
    return ids, s.gather(1, ids) * r["scale"]


def moe_ff(h, w, f):
    ids, ws = route(h, w, f["router"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, wt in zip(ids[t].tolist(), ws[t]):
            out[t] += wt * expert(h[t:t + 1], sub(w, f"e{e}."))[0]
    if f.get("shared"):
        out = out + sigmoid(lin(w["shared.sg"], h)) * expert(h, sub(w, "shared."))
    return out


def feed_forward(h, w, f):
    return clamped_ff(h, w, f["limit"]) if f["kind"] == "dense" else moe_ff(h, w, f)


# ---------------------------------------------------------------- the model
def sub(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


MIXERS = {"parallel": parallel_mixer, "attention": attention}


def forward(cfg: dict, tensors: dict, tokens, return_layers: bool = False):
    """Logits [n, vocab] of one sequence from position 0; with ``return_layers`` also the stream after every layer."""
    W = {k: v.to(F64) for k, v in tensors.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x = W["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    after = []
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        y = MIXERS[L["type"]](rms_unit(x, eps) * W[p + "norm1"], sub(W, p + "mix."), L["mixer"], eps)
        x = x + mult * rms_unit(y, eps) * W[p + "norm1b"]
        if L.get("mlp") is not None:
            y = feed_forward(rms_unit(x, eps) * W[p + "norm2"], sub(W, p + "mlp."), L["mlp"])
            x = x + mult * rms_unit(y, eps) * W[p + "norm2b"]
        after.append(x)
    logits = lin(W["embed"], rms_unit(x, eps) * W["final.norm"])
    return (logits, torch.stack(after) if after else x[None][:0]) if return_layers else logits


# ------------------------------------------------------------------ small configs and random weights
def left_half(heads=6, kv_heads=2, dim=10, vdim=7, scale=0.4, size=9, dims=6, base=700.0, factor=3.0, low=0.5, high=3.0,
              original=40, scaled=True):
    rot = {"base": base, "dims": dims}
    if scaled:
        rot["scaling"] = {"factor": factor, "low": low, "high": high, "original": original}
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": size}, "rot": rot}


def right_half(heads=4, kv_heads=2, dim=6, vdim=9, conv=3):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def parallel_layer(left=None, right=None, mlp=None):
    return {"type": "parallel", "mixer": {"left": left or left_half(), "right": right or right_half()}, "mlp": mlp}


def attention_layer(heads=4, kv_heads=2, dim=8, vdim=5, scale=0.35, coef=0.4, every=7, mlp=None):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
                      "q_temp": {"coef": coef, "every": every}}}


def dense(ff=30, limit=0.8):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts=6, top=2, ff=12, groups=(3, 2), scale=1.3, shared=18):
    f = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "scale": scale}}
    if groups:
        f["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared:
        f["shared"] = {"ff": shared}
    return f


def make_config(layers, width=28, vocab=90, eps=1e-5, scale=3.0, mult=0.4):
    return {"architecture": "Lugetar", "embedding": {"scale": scale}, "layers": layers, "norm": {"eps": eps},
            "residual_mult": mult, "vocab": vocab, "width": width}


def make_weights(cfg, seed=0, gain=1.0, rank=11):
    """Random checkpoint tensors (values representable in bf16) under the design's names."""
    gen = torch.Generator().manual_seed(seed)
    Wd = cfg["width"]

    def rnd(*shape, std=1.0):
        return torch.randn(*shape, generator=gen) * std

    def mat(o, i, k=1.0):
        return rnd(o, i, std=k * gain / math.sqrt(i))

    def attn(m, p):
        q, kk, v = m["heads"] * m["dim"], m["kv_heads"] * m["dim"], m["kv_heads"] * m["vdim"]
        return {p + "q": mat(q, Wd), p + "k": mat(kk, Wd), p + "v": mat(v, Wd), p + "q.norm": 1.5 + rnd(q, std=0.3),
                p + "k.norm": 1.5 + rnd(kk, std=0.3), p + "o": mat(Wd, m["heads"] * m["vdim"])}

    def delta(m, p):
        rank_g = rank + (8 if rank % 8 == 0 else 2)   # the two bottlenecks differ in width
        qk, v, dec, taps = m["kv_heads"] * m["dim"], m["heads"] * m["vdim"], m["heads"] * m["dim"], m["conv"]
        t = {p + "b": mat(m["heads"], Wd, 1.5), p + "A_log": rnd(m["heads"], std=0.5) - 1.5,
             p + "dt_bias": rnd(dec, std=0.7), p + "norm": 1 + rnd(m["vdim"], std=0.2), p + "a1": mat(rank, Wd),
             p + "a2": mat(dec, rank, 1.5), p + "g1": mat(rank_g, Wd), p + "g2": mat(v, rank_g, 2.0), p + "o": mat(Wd, v)}
        for n, c in (("q", qk), ("k", qk), ("v", v)):
            t[p + n], t[p + n + ".conv"] = mat(c, Wd, 1.5), rnd(c, taps, std=0.7)
        return t

    W = {"embed": rnd(cfg["vocab"], Wd, std=1.0 / cfg["embedding"]["scale"]), "final.norm": 1 + rnd(Wd, std=0.2)}
    for i, l in enumerate(cfg["layers"]):
        m, f, p = l["mixer"], l["mlp"], f"l{i}.mix."
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if f is not None else ()):
            W[f"l{i}.{n}"] = 1 + rnd(Wd, std=0.2)
        if l["type"] == "parallel":
            W.update(attn(m["left"], p + "left."))
            W.update(delta(m["right"], p + "right."))
            W[p + "left.out"], W[p + "right.out"] = 1 + rnd(Wd, std=0.3), 1 + rnd(Wd, std=0.3)
        else:
            W.update(attn(m, p))
        if f is None:
            continue
        p = f"l{i}.mlp."
        parts = {"": f["ff"]} if f["kind"] == "dense" else {f"e{e}.": f["expert"]["ff"] for e in range(f["router"]["experts"])}
        if f["kind"] == "moe":
            W[p + "router"] = mat(f["router"]["experts"], Wd, 1.5)
            if f.get("shared"):
                parts["shared."] = f["shared"]["ff"]
                W[p + "shared.sg"] = mat(1, Wd, 2.0)
        for e, ff in parts.items():
            W[p + e + "gate"], W[p + e + "up"], W[p + e + "down"] = mat(ff, Wd, 1.5), mat(ff, Wd, 1.5), mat(Wd, ff)
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
