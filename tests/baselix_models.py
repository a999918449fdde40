"""Small Baselix configurations and model folders for the tests.

The folders are written here with draws of the tests' own (not by the framework's random-weights mode): matrices
N(0, 1/in), queries a few times as large so that attention is peaked, norm weights spread visibly around zero (they are
counted from one), position vectors of the size of the tokens', sinks that take a visible share of the weight, routers
whose logits are spread out and biases that change the choice.
"""
from __future__ import annotations

import copy
import json
import math
import os
from typing import Dict, Optional

import torch


def layer(heads, dim, vdim, rank, window=None, kv_from=None, scale=None, mlp=None):
    mixer = dict(heads=heads, dim=dim, vdim=vdim, kv_rank=rank, scale=scale if scale is not None else dim ** -0.5)
    if window is not None:
        mixer["mask"] = dict(size=window)
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return dict(type="latent_attention", mixer=mixer, mlp=mlp)


def dense(ff):
    return dict(kind="dense", ff=ff)


def moe(experts, top, ff, limit, shared=None, shared_limit=None):
    return dict(kind="moe", expert=dict(ff=ff, limit=limit), router=dict(experts=experts, top=top),
                shared=dict(ff=shared, limit=shared_limit if shared_limit is not None else limit) if shared else None)


# Configurations that differ in every size and constant: one head, odd numbers of heads, more than sixteen; key, value and
# latent sizes that are no multiples of anything, that suit the matrix cores, beyond a wave, of one; latents taken over from
# the layer before, from one further back, by several layers, with windows narrower than the writer's, wider, and none;
# windows of 1 to 150 positions (inside one tile of keys, across two, no multiple of a page) and none; layers without a
# feed-forward, dense ones, one to nine experts of which one to all are chosen, with and without a shared one of another
# size and limit; a factor on the sublayers below one, one and above; a cap that bends the logits hard, hardly, and none.
CONFIGS: Dict[str, dict] = {
    "A": dict(architecture="Baselix", vocab=97, width=48, max_positions=310, norm=dict(eps=1e-5), residual_mult=0.4, logit_softcap=9.0, layers=[
        layer(3, 12, 10, 20, window=9, mlp=moe(6, 2, 24, 1.5, shared=17, shared_limit=0.8)),
        layer(4, 8, 14, 20, window=23, kv_from=0, scale=0.5, mlp=dense(70)),
        layer(2, 16, 6, 20, window=4, kv_from=0, mlp=None),
        layer(5, 6, 9, 13, window=17, mlp=moe(9, 3, 11, 3.0))]),
    # sizes of the matrix-core attention kernel throughout (one, two and four tokens a tile; more than sixteen heads)
    "B": dict(architecture="Baselix", vocab=130, width=64, max_positions=300, norm=dict(eps=1e-6), residual_mult=0.7, logit_softcap=20.0, layers=[
        layer(4, 16, 24, 32, window=40, mlp=dense(96)),
        layer(16, 8, 8, 32, window=70, kv_from=0, mlp=moe(4, 1, 32, 2.0, shared=24)),
        layer(8, 24, 16, 96, window=33, mlp=moe(5, 2, 16, 1.0)),
        layer(20, 8, 16, 96, window=150, kv_from=2, mlp=dense(64))]),
    "C": dict(architecture="Baselix", vocab=77, width=42, max_positions=260, norm=dict(eps=1e-3), residual_mult=1.0, layers=[    # no cap, m = 1
        layer(5, 7, 11, 9, window=30, scale=0.7, mlp=None),
        layer(1, 10, 5, 23, mlp=moe(5, 2, 12, 0.9, shared=30, shared_limit=4.0)),                                   # no window
        layer(3, 7, 3, 9, window=64, kv_from=0, mlp=dense(50)),
        layer(7, 3, 6, 23, window=6, kv_from=1, mlp=moe(3, 3, 10, 2.5))]),
    "D": dict(architecture="Baselix", vocab=64, width=40, max_positions=302, norm=dict(eps=1e-4), residual_mult=1.6, logit_softcap=3.0, layers=[
        layer(2, 20, 70, 68, window=65, mlp=dense(33)),
        layer(18, 4, 4, 68, kv_from=0, mlp=moe(8, 3, 8, 1.2, shared=8)),                                            # reads every key of a windowed writer
        layer(1, 130, 40, 40, window=16, mlp=dense(40))]),
    # ones and equals: a window of one key (the row's own) and of two, one head, a latent of one number, one expert in all
    "E": dict(architecture="Baselix", vocab=50, width=24, max_positions=200, norm=dict(eps=1e-6), residual_mult=0.5, logit_softcap=1.0, layers=[
        layer(1, 1, 1, 1, window=2, mlp=moe(1, 1, 8, 1.0, shared=8)),
        layer(1, 8, 8, 8, window=1, mlp=dense(8)),
        layer(8, 8, 8, 8, window=100, kv_from=1, scale=1.0, mlp=moe(2, 2, 8, 1.0, shared=8)),
        layer(1, 1, 1, 1, window=2, kv_from=0, mlp=moe(4, 1, 8, 1.0))]),
    "F": dict(architecture="Baselix", vocab=40, width=20, max_positions=140, norm=dict(eps=1e-2), residual_mult=0.05, logit_softcap=100.0, layers=[
        layer(2, 6, 10, 12, window=64, mlp=dense(20))]),
    # widths at which the products take their matrix-core forms: multiples of 64, a prompt of a few hundred rows
    "G": dict(architecture="Baselix", vocab=320, width=192, max_positions=280, norm=dict(eps=1e-5), residual_mult=0.3, logit_softcap=25.0, layers=[
        layer(6, 32, 32, 128, window=48, mlp=dense(448)),
        layer(6, 64, 32, 128, window=100, kv_from=0, mlp=moe(8, 2, 64, 1.8, shared=128)),
        layer(12, 16, 48, 64, window=130, mlp=dense(192))]),
}
SEEDS = {"A": 11, "B": 22, "C": 33, "D": 44, "E": 55, "F": 66, "G": 77}


def settled(config: dict) -> dict:
    """The configuration without what a rounding can turn, for runs in reduced precision: routers that have nothing to
    choose (every expert used, each still weighed by its logit; where a choice is a close call -- a few rows in a hundred,
    with any weights -- a rounding makes it, and the rows after it are then another model's), and no latent of one number
    (its norm leaves the number's sign, which is anyone's where the number is nearly zero)."""
    out = copy.deepcopy(config)
    for entry in out["layers"]:
        if entry["mlp"] is not None and entry["mlp"]["kind"] == "moe":
            entry["mlp"]["router"]["top"] = entry["mlp"]["router"]["experts"]
        if entry["mixer"]["kv_rank"] == 1:
            entry["mixer"]["kv_rank"] = 7
    return out


def tensors_for(config: dict, seed: int, query_factor: float = 2.0) -> Dict[str, torch.Tensor]:
    gen = torch.Generator().manual_seed(seed)

    def normal(*shape, std=1.0, mean=0.0):
        return torch.randn(*shape, generator=gen) * std + mean

    def matrix(out, inn, factor=1.0):
        return normal(out, inn, std=factor / math.sqrt(inn))
    W = config["width"]
    t = {"embed": normal(config["vocab"], W), "pos": normal(config["max_positions"], W, std=0.8), "final.norm": normal(W, std=0.2)}
    for i, entry in enumerate(config["layers"]):
        p, m = f"l{i}.", entry["mixer"]
        H, d, e, rank = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
        t[p + "norm1"] = normal(W, std=0.2)
        t[p + "mix.q"] = matrix(H * d, W, query_factor)
        if m.get("kv_from") is None:
            t[p + "mix.dkv"], t[p + "mix.dkv.norm"] = matrix(rank, W), normal(rank, std=0.2, mean=1.0)
        t[p + "mix.uk"], t[p + "mix.uv"], t[p + "mix.o"] = matrix(H * d, rank), matrix(H * e, rank), matrix(W, H * e, 1.5)
        t[p + "mix.sink"] = normal(H, mean=1.0)
        mlp = entry["mlp"]
        if mlp is None:
            continue
        t[p + "norm2"] = normal(W, std=0.2)
        if mlp["kind"] == "dense":
            t[p + "mlp.up"], t[p + "mlp.down"] = matrix(mlp["ff"], W), matrix(W, mlp["ff"])
            continue
        E = mlp["router"]["experts"]
        t[p + "mlp.router"], t[p + "mlp.router.b"] = matrix(E, W, 2.0), normal(E, std=0.7)
        units = [(f"e{j}.", mlp["expert"]["ff"]) for j in range(E)] + ([("shared.", mlp["shared"]["ff"])] if mlp.get("shared") else [])
        for name, ff in units:
            t[p + "mlp." + name + "gate"], t[p + "mlp." + name + "up"] = matrix(ff, W, 1.5), matrix(ff, W, 1.5)
            t[p + "mlp." + name + "down"] = matrix(W, ff)
    return t


def write_folder(root, name: str, dtype: str, config: Optional[dict] = None, seed: Optional[int] = None, tag: str = "", **draw) -> str:
    """config.json and model.safetensors of configuration ``name`` (or of ``config``) under ``root``."""
    from safetensors.torch import save_file
    config = config or CONFIGS[name]
    out = os.path.join(str(root), f"baselix_{name}_{dtype}{tag}")
    if not os.path.exists(os.path.join(out, "model.safetensors")):
        os.makedirs(out, exist_ok=True)
        with open(os.path.join(out, "config.json"), "w", encoding="utf-8") as fh:
            json.dump(config, fh)
        store = torch.bfloat16 if dtype == "bfloat16" else torch.float32
        tensors = tensors_for(config, SEEDS.get(name, 1) if seed is None else seed, **draw)
        save_file({k: v.to(store).contiguous() for k, v in tensors.items()}, os.path.join(out, "model.safetensors"))
    return out
