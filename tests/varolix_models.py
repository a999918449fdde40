"""Small Varolix configurations and model folders for the tests.

The folders are written here with draws of the tests' own (not by the framework's random-weights mode): matrices
N(0, 1/in), queries a few times as large so that attention is peaked, norm weights spread visibly around one, biases that
count, sinks that take a visible share of the weight, forget gates mostly open and input gates spread over both signs, so
that a matrix memory holds what it was given long ago and forgets other things at once.
"""
from __future__ import annotations

import copy
import json
import math
import os
from typing import Dict, Optional

import torch


def dense(ff):
    return dict(kind="dense", ff=ff)


def attention(heads, kv_heads, dim, vdim, rot=None, base=10000.0, scaling=None, scale=None, ff=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale if scale is not None else dim ** -0.5)
    if rot:
        m["rot"] = dict(base=base, dims=rot)
        if scaling:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return dict(type="attention", mixer=m, mlp=dense(ff) if ff else None)


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, base=10000.0, scale=None, ff=None):
    m = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank,
             scale=scale if scale is not None else (dim + rot_dim) ** -0.5, rot=dict(base=base, dims=rot_dim))
    return dict(type="latent_attention", mixer=m, mlp=dense(ff) if ff else None)


def parallel(left, right, left_scale, right_scale, temp=None, cap=10.0, ff=None):
    """``left`` (heads, kv_heads, dim, vdim), ``right`` (heads, dim, vdim), ``temp`` (coef, every)."""
    a = dict(zip(("heads", "kv_heads", "dim", "vdim"), left), scale=left[2] ** -0.5)
    if temp:
        a["q_temp"] = dict(coef=temp[0], every=temp[1])
    return dict(type="parallel", mixer=dict(left=a, left_scale=left_scale, right=dict(zip(("heads", "dim", "vdim"), right), gate_cap=cap),
                                            right_scale=right_scale), mlp=dense(ff) if ff else None)


# Configurations that differ in every size and constant: one key/value head for all, one each, groups; head sizes that are no
# multiples of anything, that suit the matrix cores, beyond a wave, of one; memories in every bucket of the scan's registers;
# rotation of a whole head, a part, one pair, none, scaled in all three ranges and not; temperatures that change with every
# position, every few, hardly ever, and none; scales of both signs and one; layers without a feed-forward; no loop, loops
# from the first layer, over the middle, over one layer, over all, of one to three passes; every order of the three kinds.
CONFIGS: Dict[str, dict] = {
    "A": dict(architecture="Varolix", vocab=97, width=48, norm=dict(eps=1e-5), loop=dict(start=0, stop=2, times=2), layers=[
        parallel((4, 2, 12, 10), (3, 8, 14), 0.7, 1.3, temp=(0.4, 7), cap=6.0, ff=70),
        attention(6, 3, 10, 14, rot=6, scaling=(8.0, 64, 8.0, 1.0), ff=50),
        latent(3, 8, 6, 10, 14, 20, ff=33)]),
    # sizes of the matrix-core kernels throughout, more than sixteen heads
    "B": dict(architecture="Varolix", vocab=130, width=64, norm=dict(eps=1e-6), loop=dict(start=2, stop=3, times=3), layers=[
        latent(20, 8, 32, 16, 24, 64, base=500.0, ff=96),
        attention(8, 2, 32, 16, rot=32, base=100.0, scaling=(4.0, 100, 20.0, 2.0), ff=64),
        parallel((8, 8, 16, 32), (4, 32, 16), 0.5, 0.9, temp=(0.2, 64), cap=15.0, ff=128)]),
    "C": dict(architecture="Varolix", vocab=77, width=42, norm=dict(eps=1e-3), layers=[          # no loop, no temperature, nothing turned
        attention(5, 1, 7, 11, scale=0.5, ff=50),
        parallel((3, 3, 9, 5), (5, 7, 11), 1.0, -0.6, cap=3.0),
        attention(2, 2, 14, 3, rot=2, base=30.0),
        latent(1, 10, 2, 5, 9, 23, ff=20)]),
    "D": dict(architecture="Varolix", vocab=64, width=40, norm=dict(eps=1e-4), loop=dict(start=1, stop=3, times=1), layers=[
        parallel((2, 1, 130, 70), (2, 70, 130), -1.2, 0.4, temp=(0.7, 1), cap=8.0, ff=33),
        latent(18, 4, 8, 4, 30, 68, ff=40),
        parallel((3, 1, 20, 150), (1, 200, 6), 0.9, 1.1, temp=(0.05, 1000), cap=20.0, ff=40)]),
    # ones and equals: one head, a memory of one channel, loops over every layer
    "E": dict(architecture="Varolix", vocab=50, width=24, norm=dict(eps=1e-6), loop=dict(start=0, stop=3, times=2), layers=[
        parallel((1, 1, 8, 8), (1, 1, 2), 1.0, 1.0, temp=(1.0, 1), cap=1.0, ff=8),
        attention(1, 1, 8, 8, rot=8, scaling=(1.0, 8, 1.0, 1.0), ff=8),
        latent(8, 8, 8, 8, 8, 8, ff=8)]),
    # widths at which the products take their matrix-core forms: multiples of 64, a prompt of a few hundred rows
    "F": dict(architecture="Varolix", vocab=320, width=192, norm=dict(eps=1e-5), loop=dict(start=1, stop=2, times=2), layers=[
        attention(6, 2, 32, 64, rot=16, scaling=(16.0, 128, 10.0, 1.0), ff=448),
        parallel((6, 2, 32, 64), (4, 64, 64), 0.6, 0.8, temp=(0.25, 50), cap=11.0, ff=256),
        latent(6, 32, 32, 32, 64, 128, ff=192)]),
}
SEEDS = {"A": 11, "B": 22, "C": 33, "D": 44, "E": 55, "F": 66}


def settled(config: dict) -> dict:
    """The configuration for runs in reduced precision: no memory of one channel or two values (their output is a direction
    among very few, which a rounding turns around wherever the sum behind it nearly vanishes)."""
    out = copy.deepcopy(config)
    for entry in out["layers"]:
        if entry["type"] == "parallel":
            right = entry["mixer"]["right"]
            right["dim"], right["vdim"] = max(right["dim"], 6), max(right["vdim"], 6)
    return out


def tensors_for(config: dict, seed: int, query_factor: float = 2.0) -> Dict[str, torch.Tensor]:
    gen = torch.Generator().manual_seed(seed)

    def normal(*shape, std=1.0, mean=0.0):
        return torch.randn(*shape, generator=gen) * std + mean

    def matrix(out, inn, factor=1.0):
        return normal(out, inn, std=factor / math.sqrt(inn))
    W = config["width"]
    t = {"embed": normal(config["vocab"], W), "head": matrix(config["vocab"], W, 2.0), "final.norm": normal(W, std=0.2, mean=1.0)}

    def heads(p, m, query):
        H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        t[p + "q"], t[p + "k"], t[p + "v"], t[p + "o"] = matrix(H * d, W, query), matrix(G * d, W), matrix(G * e, W), matrix(W, H * e, 1.5)
        t[p + "q.b"], t[p + "k.b"], t[p + "v.b"] = normal(H * d, std=0.5), normal(G * d, std=0.5), normal(G * e, std=0.3)
    for i, entry in enumerate(config["layers"]):
        p, m = f"l{i}.mix.", entry["mixer"]
        t[f"l{i}.norm1"] = normal(W, std=0.2, mean=1.0)
        if entry["type"] == "attention":
            heads(p, m, query_factor)
        elif entry["type"] == "latent_attention":
            H, d, r, e, rank, low = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"]
            t[p + "dq"], t[p + "dq.norm"], t[p + "uq"] = matrix(low, W), normal(low, std=0.2, mean=1.0), matrix(H * (d + r), low, query_factor)
            t[p + "dkv"], t[p + "dkv.norm"] = matrix(rank + r, W), normal(rank, std=0.2, mean=1.0)
            t[p + "uk"], t[p + "uv"], t[p + "sink"] = matrix(H * d, rank), matrix(H * e, rank), normal(H, mean=1.0)
            t[p + "g"], t[p + "o"] = matrix(H, W, 1.5), matrix(W, H * e, 2.0)
        else:
            left, right = m["left"], m["right"]
            heads(p + "left.", left, 1.0)
            t[p + "left.q.norm"], t[p + "left.k.norm"] = normal(left["dim"], std=0.3, mean=1.6), normal(left["dim"], std=0.3, mean=1.2)
            t[p + "left.o.b"] = normal(W, std=0.3)
            H, d, e, p = right["heads"], right["dim"], right["vdim"], p + "right."
            t[p + "q"], t[p + "k"], t[p + "v"], t[p + "g"] = matrix(H * d, W, 1.5), matrix(H * d, W), matrix(H * e, W), matrix(H * e, W)
            # A key lies near its own token's query: a head's output is brought to unit size whatever it was, and where a token's
            # own share nearly vanishes (the first token has no other) a rounding would turn the head around.
            t[p + "k"] = 0.6 * t[p + "k"] + 0.6 * t[p + "q"]
            t[p + "i"], t[p + "i.b"], t[p + "f"], t[p + "f.b"] = matrix(H, W, 2.0), normal(H, mean=-0.5), matrix(H, W, 1.5), normal(H, mean=4.0)
            t[p + "norm"], t[p + "o"] = normal(H * e, std=0.2, mean=1.0), matrix(W, H * e, 1.5)
        if entry["mlp"] is not None:
            ff = entry["mlp"]["ff"]
            t[f"l{i}.norm2"] = normal(W, std=0.2, mean=1.0)
            t[f"l{i}.mlp.gate"], t[f"l{i}.mlp.up"], t[f"l{i}.mlp.down"] = matrix(ff, W, 1.5), matrix(ff, W), matrix(W, ff)
    return t


def write_folder(root, name: str, dtype: str, config: Optional[dict] = None, seed: Optional[int] = None, **draw) -> str:
    """config.json and model.safetensors of configuration ``name`` (or of ``config``) under ``root``."""
    from safetensors.torch import save_file
    config = config or CONFIGS[name]
    out = os.path.join(str(root), f"varolix_{name}_{dtype}")
    if not os.path.exists(os.path.join(out, "model.safetensors")):
        os.makedirs(out, exist_ok=True)
        with open(os.path.join(out, "config.json"), "w", encoding="utf-8") as fh:
            json.dump(config, fh)
        store = torch.bfloat16 if dtype == "bfloat16" else torch.float32
        tensors = tensors_for(config, SEEDS.get(name, 1) if seed is None else seed, **draw)
        save_file({k: v.to(store).contiguous() for k, v in tensors.items()}, os.path.join(out, "model.safetensors"))
    return out
