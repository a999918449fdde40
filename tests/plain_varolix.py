"""A plain, slow implementation of the Varolix decoder for the tests.

Whole sequences, no cache, no state carried between calls, one function for each mechanism, written from the
design's equations and sharing no code with the engine: it reads config.json with ``json`` and the weights with
the ``safetensors`` package.  Arithmetic is float64 by default.

The design, in this file's notation (a linear weight is stored [out, in] and applied as W x; p counts a
sequence's tokens from 0; rms_e(v) = sqrt(mean(v^2) + e)):

  stream     x = E[token]; the layers start .. stop - 1 run ``times`` times in a row, then the others go on
  layer      x += A(N1(x));  x += F(N2(x))                      (a layer may have no F)
  N(v)       v / rms_e(v) w
  F          Wd (gelu(Wg h) * (Wu h)), the gelu written with tanh
  A          one of
    attention          q, k, v with biases; the first elements of a head of q and k turned by position in two halves, with
                       scaled frequencies and an amplitude if the layer says so; softmax over j <= p
    latent_attention   q = Uq (N(Dq h)); one latent c = N((D h)[:rank]) and one turned key part (D h)[rank:] a token; per
                       head k = [Uk c | turned part], v = Uv c; softmax with a sink; a head's sum times sigmoid(Wg h)_head
    parallel           a L(h) + b M(h).  L: attention that turns nothing: q and k normed per head with a weight, q times
                       1 + c ln(floor((p + 1) / n) + 1), biases on q, k, v and the output.  M: a matrix memory per head,
                         m_t = max(f_t + m_(t-1), i_t)               m, S, n from zero
                         S_t = e^(f_t + m_(t-1) - m_t) S_(t-1) + e^(i_t - m_t) k_t v_t^T,  n_t likewise with k_t alone
                         o_t = S_t^T q_t / (max(|n_t . q_t|, e^(-m_t)) + 1e-6), over rms_e(o_t), times a weight and sigmoid(Wg h)
                       with log gates i = C tanh((Wi h + bi) / C) and f = log sigmoid(C tanh((Wf h + bf) / C))
  logits     W_head N(x)
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


def rms_norm(v: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return unit_rms(v, eps) * w


def gelu_by_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def turning_speeds(dims: int, base: float, scaling: Optional[dict] = None):
    """(what pair i turns by a position, for i < dims / 2; the factor on cosines and sines)."""
    speeds = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if scaling is None:
        return torch.tensor(speeds, dtype=torch.float64), 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])

    def index_of(turns: float) -> float:
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(index_of(float(scaling["fast"]))), 0)
    hi = min(math.ceil(index_of(float(scaling["slow"]))), dims - 1)
    out = []
    for i, f in enumerate(speeds):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / factor * ramp + f * (1.0 - ramp))
    return torch.tensor(out, dtype=torch.float64), 0.1 * math.log(factor) + 1.0


def turn_halves(v: torch.Tensor, positions: torch.Tensor, speeds: torch.Tensor, amplitude: float = 1.0) -> torch.Tensor:
    """v [T, ..., d]: element i of the first 2 n (n speeds) is paired with element i + n; the rest passes."""
    n = speeds.numel()
    shape = [v.shape[0]] + [1] * (v.dim() - 2) + [n]
    angle = (positions.to(torch.float64)[:, None] * speeds[None, :]).reshape(shape)
    c, s = (torch.cos(angle) * amplitude).to(v.dtype), (torch.sin(angle) * amplitude).to(v.dtype)
    a, b = v[..., :n], v[..., n:2 * n]
    return torch.cat([a * c - b * s, b * c + a * s, v[..., 2 * n:]], dim=-1)


def query_temperature(positions: torch.Tensor, coef: float, every: float) -> torch.Tensor:
    """The factor on a query at each position."""
    return torch.tensor([1.0 + coef * math.log(math.floor((int(p) + 1) / every) + 1.0) for p in positions], dtype=torch.float64)


def causal_weights(scores: torch.Tensor, sink: Optional[torch.Tensor] = None) -> torch.Tensor:
    """scores [heads, T, T] -> softmax over j <= i, with exp(sink_head) in the denominator if there is a sink."""
    T = scores.shape[-1]
    s = scores.masked_fill(~torch.tril(torch.ones(T, T, dtype=torch.bool)), -math.inf)
    top = s.max(dim=-1, keepdim=True).values
    if sink is not None:
        top = torch.maximum(top, sink[:, None, None])
    e = torch.exp(s - top)
    total = e.sum(dim=-1, keepdim=True)
    if sink is not None:
        total = total + torch.exp(sink[:, None, None] - top)
    return e / total


def grouped_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, sink: Optional[torch.Tensor] = None) -> torch.Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, e] -> [T, H, e]; head a reads key/value head a // (H / G)."""
    H, G = q.shape[1], k.shape[1]
    of = [a // (H // G) for a in range(H)]
    s = torch.stack([q[:, a] @ k[:, of[a]].T for a in range(H)]) * scale
    w = causal_weights(s, sink)
    return torch.stack([w[a] @ v[:, of[a]] for a in range(H)], dim=1)


def log_input_gate(z: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(z / cap)


def log_forget_gate(z: torch.Tensor, cap: float) -> torch.Tensor:
    return torch.nn.functional.logsigmoid(cap * torch.tanh(z / cap))


def matrix_memory(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, i: torch.Tensor, f: torch.Tensor, state=None):
    """One head: q, k [T, d], v [T, e], log gates i, f [T] -> (o [T, e], (S, n, m) after the last token)."""
    T, d = q.shape
    if state is None:
        state = torch.zeros(d, v.shape[1], dtype=q.dtype), torch.zeros(d, dtype=q.dtype), torch.zeros((), dtype=q.dtype)
    S, n, m = state
    out = torch.zeros(T, v.shape[1], dtype=q.dtype)
    for t in range(T):
        top = torch.maximum(f[t] + m, i[t])
        keep, add = torch.exp(f[t] + m - top), torch.exp(i[t] - top)
        S = keep * S + add * torch.outer(k[t], v[t])
        n = keep * n + add * k[t]
        m = top
        out[t] = (S.T @ q[t]) / (torch.maximum((n @ q[t]).abs(), torch.exp(-m)) + 1e-6)
    return out, (S, n, m)


# --- the model ---------------------------------------------------------------------

class PlainVarolix:
    def __init__(self, folder: str, dtype: torch.dtype = torch.float64, rounded: bool = False):
        """``rounded``: what goes into a linear map and what comes out is rounded to bfloat16 (how far rounding alone moves a row)."""
        from safetensors.torch import load_file
        with open(os.path.join(folder, "config.json"), encoding="utf-8") as fh:
            self.cfg = json.load(fh)
        self.dtype, self.rounded = dtype, rounded
        self.w: Dict[str, torch.Tensor] = {k: v.to(dtype) for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}
        self.eps = float(self.cfg["norm"]["eps"])

    def lin(self, name: str, h: torch.Tensor, bias: bool = False) -> torch.Tensor:
        if self.rounded:
            h = h.to(torch.bfloat16).to(self.dtype)
        y = h @ self.w[name].T + (self.w[name + ".b"] if bias else 0.0)
        return y.to(torch.bfloat16).to(self.dtype) if self.rounded else y

    def attention(self, p: str, m: dict, h: torch.Tensor, pos: torch.Tensor) -> torch.Tensor:
        T, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        q, k = self.lin(p + "q", h, True).view(T, H, d), self.lin(p + "k", h, True).view(T, G, d)
        v = self.lin(p + "v", h, True).view(T, G, e)
        rot = m.get("rot")
        if rot is not None:
            speeds, amplitude = turning_speeds(rot["dims"], rot["base"], rot.get("scaling"))
            q, k = turn_halves(q, pos, speeds, amplitude), turn_halves(k, pos, speeds, amplitude)
        return self.lin(p + "o", grouped_attention(q, k, v, m["scale"]).reshape(T, H * e))

    def latent_attention(self, p: str, m: dict, h: torch.Tensor, pos: torch.Tensor) -> torch.Tensor:
        w, T, H, d, r, e, rank = self.w, h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
        q = self.lin(p + "uq", rms_norm(self.lin(p + "dq", h), w[p + "dq.norm"], self.eps)).view(T, H, d + r)
        both = self.lin(p + "dkv", h)
        c = rms_norm(both[:, :rank], w[p + "dkv.norm"], self.eps)
        speeds, _ = turning_speeds(m["rot"]["dims"], m["rot"]["base"])
        q = torch.cat([q[..., :d], turn_halves(q[..., d:], pos, speeds)], dim=-1)
        turned = turn_halves(both[:, rank:], pos, speeds)[:, None].expand(T, H, r)
        k = torch.cat([self.lin(p + "uk", c).view(T, H, d), turned], dim=-1)
        o = grouped_attention(q, k, self.lin(p + "uv", c).view(T, H, e), m["scale"], w[p + "sink"])
        return self.lin(p + "o", (o * torch.sigmoid(self.lin(p + "g", h))[:, :, None]).reshape(T, H * e))

    def normed_attention(self, p: str, m: dict, h: torch.Tensor, pos: torch.Tensor) -> torch.Tensor:
        w, T, H, G, d, e = self.w, h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        q = rms_norm(self.lin(p + "q", h, True).view(T, H, d), w[p + "q.norm"], self.eps)
        k = rms_norm(self.lin(p + "k", h, True).view(T, G, d), w[p + "k.norm"], self.eps)
        if m.get("q_temp") is not None:
            q = q * query_temperature(pos, m["q_temp"]["coef"], m["q_temp"]["every"]).to(q.dtype)[:, None, None]
        o = grouped_attention(q, k, self.lin(p + "v", h, True).view(T, G, e), m["scale"])
        return self.lin(p + "o", o.reshape(T, H * e), True)

    def memory(self, p: str, m: dict, h: torch.Tensor) -> torch.Tensor:
        T, H, d, e, cap = h.shape[0], m["heads"], m["dim"], m["vdim"], float(m["gate_cap"])
        q, k = (self.lin(p + "q", h) * d ** -0.5).view(T, H, d), self.lin(p + "k", h).view(T, H, d)
        v = self.lin(p + "v", h).view(T, H, e)
        # (the gates' logits are not rounded: they enter the recurrence)
        zi, zf = (h @ self.w[p + n].T + self.w[p + n + ".b"] for n in ("i", "f"))
        i, f = log_input_gate(zi, cap), log_forget_gate(zf, cap)
        o = torch.stack([matrix_memory(q[:, a], k[:, a], v[:, a], i[:, a], f[:, a])[0] for a in range(H)], dim=1)
        o = unit_rms(o, self.eps).reshape(T, H * e) * self.w[p + "norm"] * torch.sigmoid(self.lin(p + "g", h))
        return self.lin(p + "o", o)

    def mixer(self, kind: str, p: str, m: dict, h: torch.Tensor, pos: torch.Tensor) -> torch.Tensor:
        if kind == "attention":
            return self.attention(p, m, h, pos)
        if kind == "latent_attention":
            return self.latent_attention(p, m, h, pos)
        assert kind == "parallel"
        return (m["left_scale"] * self.normed_attention(p + "left.", m["left"], h, pos)
                + m["right_scale"] * self.memory(p + "right.", m["right"], h))

    def order(self) -> List[int]:
        n, loop = len(self.cfg["layers"]), self.cfg.get("loop")
        if loop is None:
            return list(range(n))
        inner = list(range(loop["start"], loop["stop"]))
        return list(range(loop["start"])) + inner * loop["times"] + list(range(loop["stop"], n))

    def forward(self, ids: Sequence[int], return_layers: bool = False):
        """float logits [T, vocab] of one sequence from its first token (and, if asked, the stream after every layer run)."""
        w = self.w
        pos = torch.arange(len(ids))
        x, after = w["embed"][torch.as_tensor(list(ids), dtype=torch.long)], []
        for n in self.order():
            layer, p = self.cfg["layers"][n], f"l{n}."
            x = x + self.mixer(layer["type"], p + "mix.", layer["mixer"], rms_norm(x, w[p + "norm1"], self.eps), pos)
            if layer.get("mlp") is not None:
                assert layer["mlp"]["kind"] == "dense"
                h = rms_norm(x, w[p + "norm2"], self.eps)
                x = x + self.lin(p + "mlp.down", gelu_by_tanh(self.lin(p + "mlp.gate", h)) * self.lin(p + "mlp.up", h))
            after.append(x.clone())
        logits = self.lin("head", rms_norm(x, w["final.norm"], self.eps)).to(torch.float32)
        return (logits, after) if return_layers else logits
