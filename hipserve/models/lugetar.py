"""Lugetar: a layer-list decoder (``config.LugetarConfig``) with a norm before and a norm after every sublayer,

    x <- x + m * norm1b(mixer(norm1(x)));   x <- x + m * norm2b(ff(norm2(x)))

(the second only where the layer has a feed-forward) and one multiplier m for the whole model. Mixers
(``models/mixers.py``): chunked attention beside a gated delta rule with a decay per key channel, each half's
output normed over the width before they are averaged; or plain causal attention whose queries grow with
their position. Feed-forwards: dense with a clamped gate, or routed gated experts with a gated shared expert.
The embedding is scaled, the logits read the unscaled table.

The residual stream lives in 32-bit floats for every dtype. One fused op (``sandwich_update``) sits between two
sublayers: the sublayer's result put together (the two normed halves of a parallel mixer, or the experts' rows
and the shared expert), its norm, the sum into the stream and the next sublayer's norm. The first one reads the
embedding table itself.
"""
from __future__ import annotations

import torch

from .layer_list import LayerListModel
from .mixers import RoutedMoE


class LugetarModel(LayerListModel):
    norm_library = "delta"

    # ---------------------------------------------------------------- weights
    def load_tensors(self, get):
        """Names as in ``LayerListModel.load_tensors`` without ``head`` (the embedding table serves), and
        ``l<i>.norm1b`` / ``.norm2b``, the norms of the sublayers' results."""
        dev, dt = self.device, self.dtype
        self.embed = self.lm_head = get("embed").to(dev, dt).contiguous()
        self.final_norm = get("final.norm").to(dev, torch.float32)
        for i, lw in enumerate(self.layers):
            lw.norm1, lw.norm1b = (get(f"l{i}.{n}").to(dev, torch.float32) for n in ("norm1", "norm1b"))
            lw.mixer.load(get, f"l{i}.mix.")
            if lw.mlp is not None:
                lw.norm2, lw.norm2b = (get(f"l{i}.{n}").to(dev, torch.float32) for n in ("norm2", "norm2b"))
                lw.mlp.load(get, f"l{i}.mlp.")

    def random_tensors(self, seed: int = 0, std: float = 0.05) -> dict:
        cfg = self.cfg
        g = torch.Generator().manual_seed(seed)
        H, V = cfg.hidden_size, cfg.vocab_size
        out = {"embed": torch.randn(V, H, generator=g) / max(cfg.embed_scale, 1e-6),
               "final.norm": 1.0 + 0.1 * torch.randn(H, generator=g)}
        for i, lw in enumerate(self.layers):
            for n in ("norm1", "norm1b") + (("norm2", "norm2b") if lw.mlp is not None else ()):
                out[f"l{i}.{n}"] = 1.0 + 0.1 * torch.randn(H, generator=g)
            for k, v in lw.mixer.init_random(g, std).items():
                out[f"l{i}.mix.{k}"] = v
            if lw.mlp is not None:
                for k, v in lw.mlp.init_random(g, std).items():
                    out[f"l{i}.mlp.{k}"] = v
        return {k: v.bfloat16().float() for k, v in out.items()}

    def step_workspace_bytes(self, tokens: int, seqs: int) -> int:
        return super().step_workspace_bytes(tokens, seqs) + tokens * self.cfg.hidden_size * 24

    # ---------------------------------------------------------------- forward
    def forward(self, ids: torch.Tensor, meta, kv_caches) -> torch.Tensor:
        ops, cfg = self.ops, self.cfg
        T, H = ids.shape[0], cfg.hidden_size
        state = meta.state
        if meta.id_src is not None:  # decode lookahead: row i's id is the previous step's sample tok[src[i]]
            src, tok = meta.id_src
            ids = torch.where(src >= 0, tok.index_select(0, src.clamp(min=0)), ids)
        residual = torch.empty(T, H, device=ids.device, dtype=torch.float32)

        def update(norm, post=None, y=None, table=None):
            out = torch.empty(T, H, device=ids.device, dtype=self.dtype)
            return ops.sandwich_update(out, residual, norm, cfg.norm_eps, y, post, cfg.residual_mult, table)

        def first_norm(r):
            return self.final_norm if r == len(self.runs) else self.layers[self.runs[r][0]].norm1

        h = update(first_norm(0), table=(self.embed, ids, cfg.embed_scale))
        for r, (i, _, _) in enumerate(self.runs):
            lw = self.layers[i]
            y = lw.mixer.forward(h, meta, kv_caches[r], state[r] if state is not None else None)
            if lw.mlp is not None:
                h = update(lw.norm2, lw.norm1b, y)
                y = lw.mlp.forward(h)
                if isinstance(lw.mlp, RoutedMoE):
                    ye, pair_slot, _, wts, _, _, shared = y
                    y = (ye, pair_slot, wts, shared, lw.mlp.shared_gate if shared is not None else None)
                h = update(first_norm(r + 1), lw.norm2b, y)
            else:
                h = update(first_norm(r + 1), lw.norm1b, y)
            if self.capture is not None:
                self.capture.append(residual.clone())
        return h
