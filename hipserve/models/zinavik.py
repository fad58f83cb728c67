"""Zinavik: a layer-list decoder (``config.ZinavikConfig``) with several residual streams mixed
between the sublayers (static hyper-connections),

    u = sum_s in[s] x_s;   y = sublayer(norm(u));   x_t <- sum_s mix[s, t] x_s + out[t] y

with tensors of their own for the mixer (``hc1``) and the feed-forward (``hc2``) of every layer. The
streams all start as the scaled embedding, the logits read their sum through the (unscaled) embedding
table. The mixer of every layer (``models/mixers.py``) runs windowed attention and lightning attention side
by side; the feed-forward is a mixture of clamped gated experts, or there is none. A span of layers can
run several passes with the same weights and a cache / state per pass.

The streams live in 32-bit floats for every dtype, as [tokens, streams, width]. One fused op
(``stream_update``) sits between two sublayers: the streams' update, the next sublayer's input and its norm.
Both updates of a layer are linear in the streams, so the one after the mixer is not written back: the op
forms the updated streams in registers for the feed-forward's input only, and the op after the feed-forward
applies both updates at once,

    x <- (mix1 mix2)^T x + (mix2^T out1) y1 + out2 y2,

with the products of the small matrices taken once at load. The streams are then read twice and written
once per layer, instead of read and written twice.
"""
from __future__ import annotations

import torch

from .layer_list import LayerListModel
from .mixers import RoutedMoE


class ZinavikModel(LayerListModel):
    norm_library = "stream"

    # ---------------------------------------------------------------- weights
    def load_tensors(self, get):
        """Names as in ``LayerListModel.load_tensors`` without ``head`` (the embedding table serves), and
        ``l<i>.hc1`` / ``.hc2`` with ``.in`` [streams], ``.out`` [streams], ``.mix`` [streams, streams] (from, to)."""
        dev, dt = self.device, self.dtype
        self.embed = self.lm_head = get("embed").to(dev, dt).contiguous()
        self.final_norm = get("final.norm").to(dev, torch.float32)
        hc = {}
        for i, lw in enumerate(self.layers):
            lw.norm1 = get(f"l{i}.norm1").to(dev, torch.float32)
            lw.mixer.load(get, f"l{i}.mix.")
            if lw.mlp is not None:
                lw.norm2 = get(f"l{i}.norm2").to(dev, torch.float32)
                lw.mlp.load(get, f"l{i}.mlp.")
            hc[i] = [{k: get(f"l{i}.hc{q}.{k}").double() for k in ("in", "out", "mix")}
                     for q in ((1, 2) if lw.mlp is not None else (1,))]
        self._set_streams(hc)

    def _set_streams(self, hc: dict):
        """The coefficients of every ``stream_update`` launch: before the first run, and per run the one between
        its sublayers (None without a feed-forward) and the one after it, which also forms the next run's input."""
        S, dev = self.cfg.streams, self.device
        one, zero = torch.ones(S, dtype=torch.float64), torch.zeros(S, dtype=torch.float64)

        def pack(M, p1, p2, c):
            return torch.cat([M.reshape(-1), p1, p2, c]).to(torch.float32).to(dev).contiguous()

        def first_in(r):
            return hc[self.runs[r][0]][0]["in"] if r < len(self.runs) else one

        self.coef0 = pack(torch.eye(S, dtype=torch.float64), zero, zero, first_in(0))
        self.coefs = []
        for r, (i, _, _) in enumerate(self.runs):
            a, nxt = hc[i][0], first_in(r + 1)
            if len(hc[i]) == 1:
                self.coefs.append((None, pack(a["mix"], a["out"], zero, nxt)))
                continue
            b = hc[i][1]
            self.coefs.append((pack(a["mix"], a["out"], zero, b["in"]),
                               pack(a["mix"] @ b["mix"], a["out"] @ b["mix"], b["out"], nxt)))

    def random_tensors(self, seed: int = 0, std: float = 0.05) -> dict:
        cfg = self.cfg
        g = torch.Generator().manual_seed(seed)
        H, V, S = cfg.hidden_size, cfg.vocab_size, cfg.streams
        out = {"embed": torch.randn(V, H, generator=g) / max(cfg.embed_scale, 1e-6),
               "final.norm": 1.0 + 0.1 * torch.randn(H, generator=g)}
        for i, lw in enumerate(self.layers):
            for k, v in lw.mixer.init_random(g, std).items():
                out[f"l{i}.mix.{k}"] = v
            if lw.mlp is not None:
                for k, v in lw.mlp.init_random(g, std).items():
                    out[f"l{i}.mlp.{k}"] = v
            for q in (1, 2) if lw.mlp is not None else (1,):
                out[f"l{i}.norm{q}"] = 1.0 + 0.1 * torch.randn(H, generator=g)
                out[f"l{i}.hc{q}.in"] = 1.0 / S + 0.2 * torch.randn(S, generator=g)
                out[f"l{i}.hc{q}.out"] = 1.0 + 0.2 * torch.randn(S, generator=g)
                out[f"l{i}.hc{q}.mix"] = torch.eye(S) + 0.1 * torch.randn(S, S, generator=g)
        return {k: v.bfloat16().float() for k, v in out.items()}

    def step_workspace_bytes(self, tokens: int, seqs: int) -> int:
        return super().step_workspace_bytes(tokens, seqs) + tokens * self.cfg.hidden_size * 4 * (self.cfg.streams + 4)

    # ---------------------------------------------------------------- forward
    def forward(self, ids: torch.Tensor, meta, kv_caches) -> torch.Tensor:
        ops, cfg = self.ops, self.cfg
        T, H = ids.shape[0], cfg.hidden_size
        state = meta.state
        if meta.id_src is not None:  # decode lookahead: row i's id is the previous step's sample tok[src[i]]
            src, tok = meta.id_src
            ids = torch.where(src >= 0, tok.index_select(0, src.clamp(min=0)), ids)
        streams = torch.empty(T, cfg.streams, H, device=ids.device, dtype=torch.float32)
        # the streams' current value: all of them are the scaled embedding until the first layer's updates
        x = (self.embed, ids, cfg.embed_scale)

        def norm_of(r):
            return self.final_norm if r == len(self.runs) else self.layers[self.runs[r][0]].norm1

        h = ops.stream_update(torch.empty(T, H, device=ids.device, dtype=self.dtype), None, x, self.coef0, norm_of(0),
                              cfg.norm_eps)
        for r, (i, _, _) in enumerate(self.runs):
            lw = self.layers[i]
            mid, end = self.coefs[r]
            y1 = lw.mixer.forward(h, meta, kv_caches[r], state[r] if state is not None else None)
            y2 = None
            if lw.mlp is not None:
                h = ops.stream_update(torch.empty_like(h), None, x, mid, lw.norm2, cfg.norm_eps, y1)
                y2 = lw.mlp.forward(h)
                if isinstance(lw.mlp, RoutedMoE):
                    ye, pair_slot, _, wts, _, _, shared = y2
                    if lw.mlp.spec.weight_input:
                        wts = lw.mlp.spec.top   # applied already
                    y2 = (ye, pair_slot, wts, shared, lw.mlp.shared_gate if shared is not None else None)
            # after the last run only the sum of the streams is read: nothing is written back
            dst = streams if r + 1 < len(self.runs) or self.capture is not None else None
            h = ops.stream_update(torch.empty_like(h), dst, x, end, norm_of(r + 1), cfg.norm_eps, y1, y2)
            x = streams
            if self.capture is not None:
                self.capture.append(streams.sum(1))
        return h
