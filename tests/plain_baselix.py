"""A plain, slow implementation of the Baselix decoder for the tests.

Whole sequences, no cache, no state carried between calls, one function for each mechanism, written from the
design's equations and sharing no code with the engine: it reads config.json with ``json`` and the weights with
the ``safetensors`` package.  Arithmetic is float64 by default.

The design, in this file's notation (a linear weight is stored [out, in] and applied as W x; p counts a
sequence's tokens from 0):

  stream     x = E[token] + P[p]                                (P: a learned vector for each position)
  layer      x += m A(N1(x));  x += m F(N2(x))                  (m: one number for the whole model; a layer may have no F)
  N(v)       v / sqrt(mean(v^2) + eps) (1 + w)
  A          q = Wq h in heads; c = D h / sqrt(mean((D h)^2) + eps) g -- one latent a token for all heads --, or, in
             a layer that names another one, that layer's c; per head k = Wk c, v = Wv c; position i weighs the
             positions i - n + 1 .. i (n: the layer's window) by exp(scale q.k) / (exp(s) + sum), s a number a head;
             the heads' sums side by side through Wo
  F          dense: Wd max(Wu h, 0)^2; or experts: z = R h + b, the ``top`` largest z are chosen and weighed by the
             softmax over the chosen z alone; a unit is Wd (g sigmoid(1.702 g) (u + 1)) with g = min(Wg h, L) and
             u = Wu h held within -L..L; one more unit with sizes of its own is added for every token
  logits     C tanh(E N(x) / C)                                 (E: the table of the input)
"""
from __future__ import annotations

import json
import math
import os
from typing import Dict, List, Optional, Sequence

import torch


# --- mechanisms -----------------------------------------------------------------

def unit_rms(v: torch.Tensor, eps: float) -> torch.Tensor:
    """v / sqrt(mean(v^2) + eps) over the last axis."""
    return v / torch.sqrt((v * v).mean(dim=-1, keepdim=True) + eps)


def norm_about_one(v: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return unit_rms(v, eps) * (1.0 + w)


def placed_embedding(table: torch.Tensor, places: torch.Tensor, ids: Sequence[int], first: int = 0) -> torch.Tensor:
    """Rows of ``table`` for the ids, each plus the row of ``places`` for its position (the first id's is ``first``)."""
    return torch.stack([table[int(t)] + places[first + i] for i, t in enumerate(ids)])


def latent_of(h: torch.Tensor, down: torch.Tensor, g: torch.Tensor, eps: float) -> torch.Tensor:
    return unit_rms(h @ down.T, eps) * g


def window_mask(n: int, size: int) -> torch.Tensor:
    """[n, n] bool: row i sees column j with 0 <= i - j < size (size 0: every j <= i)."""
    i = torch.arange(n)[:, None]
    j = torch.arange(n)[None, :]
    return (j <= i) & (i - j < size if size else j <= i)


def sink_softmax(scores: torch.Tensor, mask: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """scores [heads, T, T] -> exp(s_j) / (exp(sink_head) + sum over the visible j of exp(s_j)), zero where not visible."""
    s = scores.masked_fill(~mask, -math.inf)
    top = torch.maximum(s.max(dim=-1, keepdim=True).values, sink[:, None, None])
    e = torch.exp(s - top)
    return e / (torch.exp(sink[:, None, None] - top) + e.sum(dim=-1, keepdim=True))


def latent_attention(q: torch.Tensor, c: torch.Tensor, up_k: torch.Tensor, up_v: torch.Tensor, sink: torch.Tensor, scale: float,
                     window: int) -> torch.Tensor:
    """q [T, heads, d], c [T, rank] -> [T, heads * e]; keys and values are made for every head (nothing is absorbed)."""
    T, H, d = q.shape
    k = (c @ up_k.T).reshape(T, H, d)
    v = (c @ up_v.T).reshape(T, H, -1)
    s = torch.stack([q[:, a] @ k[:, a].T for a in range(H)]) * scale
    w = sink_softmax(s, window_mask(T, window), sink)
    return torch.cat([w[a] @ v[:, a] for a in range(H)], dim=-1)


def squared_relu(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0.0) ** 2


def clamped_unit(g: torch.Tensor, u: torch.Tensor, limit: float) -> torch.Tensor:
    g, u = torch.clamp(g, max=limit), torch.clamp(u, min=-limit, max=limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def route(z: torch.Tensor, top: int):
    """z [T, E] -> (chosen [T, top], weights [T, top], margin [T]): the ``top`` largest z, weighed by the softmax over
    those alone.  margin: how far the last chosen z lies above the best one left out (inf if none is left out)."""
    order = torch.argsort(z, dim=-1, descending=True, stable=True)
    ranked = torch.gather(z, 1, order)
    weights = torch.softmax(ranked[:, :top], dim=-1)
    margin = ranked[:, top - 1] - ranked[:, top] if top < z.shape[1] else torch.full((z.shape[0],), math.inf, dtype=z.dtype)
    return order[:, :top], weights, margin


def capped(z: torch.Tensor, cap: Optional[float]) -> torch.Tensor:
    return cap * torch.tanh(z / cap) if cap else z


# --- the model ---------------------------------------------------------------------

class PlainBaselix:
    def __init__(self, folder: str, dtype: torch.dtype = torch.float64):
        from safetensors.torch import load_file
        with open(os.path.join(folder, "config.json"), encoding="utf-8") as fh:
            self.cfg = json.load(fh)
        self.dtype = dtype
        self.w: Dict[str, torch.Tensor] = {k: v.to(dtype) for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}
        self.eps = float(self.cfg["norm"]["eps"])
        self.margins: List[torch.Tensor] = []

    def mixer(self, i: int, m: dict, h: torch.Tensor, latents: Dict[int, torch.Tensor]) -> torch.Tensor:
        w, p = self.w, f"l{i}.mix."
        if m.get("kv_from") is None:
            c = latents[i] = latent_of(h, w[p + "dkv"], w[p + "dkv.norm"], self.eps)
        else:
            c = latents[m["kv_from"]]
        q = (h @ w[p + "q"].T).reshape(h.shape[0], m["heads"], m["dim"])
        window = m["mask"]["size"] if m.get("mask") else 0
        return latent_attention(q, c, w[p + "uk"], w[p + "uv"], w[p + "sink"], m["scale"], window) @ w[p + "o"].T

    def unit(self, p: str, h: torch.Tensor, limit: float) -> torch.Tensor:
        w = self.w
        return clamped_unit(h @ w[p + "gate"].T, h @ w[p + "up"].T, limit) @ w[p + "down"].T

    def feed_forward(self, p: str, mlp: dict, h: torch.Tensor) -> torch.Tensor:
        w = self.w
        if mlp["kind"] == "dense":
            return squared_relu(h @ w[p + "up"].T) @ w[p + "down"].T
        assert mlp["kind"] == "moe"
        z = h.to(torch.float64) @ w[p + "router"].to(torch.float64).T + w[p + "router.b"].to(torch.float64)
        chosen, weights, margin = route(z, mlp["router"]["top"])
        self.margins.append(margin)
        out = torch.zeros_like(h)
        for e in range(mlp["router"]["experts"]):
            rows, slot = torch.nonzero(chosen == e, as_tuple=True)
            if len(rows):
                out[rows] += weights[rows, slot, None].to(h.dtype) * self.unit(p + f"e{e}.", h[rows], mlp["expert"]["limit"])
        if mlp.get("shared"):
            out = out + self.unit(p + "shared.", h, mlp["shared"]["limit"])
        return out

    def forward(self, ids: Sequence[int], return_layers: bool = False):
        """float logits [T, vocab] of one sequence from its first token (and, if asked, the stream after every layer)."""
        w, cfg = self.w, self.cfg
        m = float(cfg["residual_mult"])
        self.margins = []
        x, after, latents = placed_embedding(w["embed"], w["pos"], ids), [], {}
        for i, layer in enumerate(cfg["layers"]):
            assert layer["type"] == "latent_attention"
            p = f"l{i}."
            x = x + m * self.mixer(i, layer["mixer"], norm_about_one(x, w[p + "norm1"], self.eps), latents)
            if layer.get("mlp") is not None:
                x = x + m * self.feed_forward(p + "mlp.", layer["mlp"], norm_about_one(x, w[p + "norm2"], self.eps))
            after.append(x.clone())
        logits = capped(norm_about_one(x, w["final.norm"], self.eps) @ w["embed"].T, cfg.get("logit_softcap")).to(torch.float32)
        return (logits, after) if return_layers else logits

    def closest_call(self) -> Optional[torch.Tensor]:
        """[T]: the smallest routing margin of every token over all routers of the last forward (None without routers)."""
        return torch.stack(self.margins).min(dim=0).values if self.margins else None
