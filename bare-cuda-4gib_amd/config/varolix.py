"""Configuration of the Varolix decoder: a stack of pre-norm layers (plain RMS norms) that each name their mixer, and a dense
feed-forward gated by the gelu written with tanh, or none.  A run of neighbouring layers may be gone through several times
with the same weights, a cache for every pass.

``attention``         q, k, v with biases, the first ``rot.dims`` elements of a head of q and k turned by position in two halves
                      (``rot.scaling``: frequencies scaled between ``fast`` and ``slow``, with an amplitude), softmax over all keys.
``latent_attention``  queries from a latent of their own (``q_rank``), one low-rank latent and one turned key part a token for all
                      heads, a sink in the softmax, a gate a head.
``parallel``          the sum of two mixers of one input, each times a constant: attention without positions but in a
                      temperature on the queries that grows with the position (``q_temp``), queries and keys normed per head,
                      biases on the projections and the output; and a matrix memory with exponential gates capped by
                      ``gate_cap`` and a normaliser.

config.json keys: ``vocab``, ``width``, ``norm.eps``, ``loop`` (``start``, ``stop``, ``times``; optional) and ``layers``, a list of
``{"type": ..., "mixer": {...}, "mlp": {"kind": "dense", "ff": N} | null}``.  A mixer of ``attention`` names ``heads``, ``kv_heads``,
``dim``, ``vdim``, ``scale`` and ``rot`` (``base``, ``dims``, ``scaling``: ``factor``, ``original``, ``fast``, ``slow``; both optional); of
``latent_attention`` ``heads``, ``dim``, ``rot_dim``, ``vdim``, ``q_rank``, ``kv_rank``, ``scale``, ``rot`` (``base``, ``dims``); of ``parallel``
``left`` (as ``attention``, with ``q_temp``: ``coef``, ``every``; optional), ``left_scale``, ``right`` (``heads``, ``dim``, ``vdim``, ``gate_cap``),
``right_scale``.
Tensor names: ``embed``, ``head``, ``final.norm``, and for layer i ``l<i>.norm1``, ``l<i>.norm2``, ``l<i>.mlp.{gate,up,down}``, under
``l<i>.mix.`` ``q,k,v,o,q.b,k.b,v.b`` (``attention``), ``dq,dq.norm,uq,dkv,dkv.norm,uk,uv,sink,g,o`` (``latent_attention``),
``left.{q,k,v,o,q.b,k.b,v.b,o.b,q.norm,k.norm}`` and ``right.{q,k,v,g,i,i.b,f,f.b,norm,o}`` (``parallel``).
"""
from __future__ import annotations

import dataclasses
from typing import Any, Dict, List, Optional, Tuple

from ..errors import ConfigError
from .base import ModelConfig, field_from_json
from .milenex import _number, _object
from .registry import Architecture, register_architecture

_ATTENTION_SIZES = ("heads", "kv_heads", "dim", "vdim")
_LATENT_SIZES = ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank")
_MEMORY_SIZES = ("heads", "dim", "vdim")


def _sizes(where: str, m: Dict[str, Any], keys) -> Dict[str, int]:
    missing = [k for k in keys if k not in m]
    if missing:
        raise ConfigError(f"config.json: {where} lacks {', '.join(missing)}")
    return {k: _number(where, m, k) for k in keys}


def _rotation(where: str, m: Dict[str, Any]):
    """The mixer's ``rot`` as the parameters of a rotary part with the rotate-half pairing (None: nothing is turned)."""
    rot = _object(where, m, "rot", required=False)
    dims = _number(where + ".rot", rot, "dims") if rot is not None else 0
    if dims == 0:
        return None
    out = dict(theta=_number(where + ".rot", rot, "base", integer=False), dim=dims)
    scaling = _object(where + ".rot", rot, "scaling", required=False)
    if scaling is not None:
        out["scaling"] = {k: _number(where + ".rot.scaling", scaling, k, integer=False) for k in ("factor", "original", "fast", "slow")}
    return out


def _attention(where: str, m: Dict[str, Any]) -> Dict[str, Any]:
    return dict(_sizes(where, m, _ATTENTION_SIZES), scale=_number(where, m, "scale", integer=False), bias=True, sink=False)


def _normed_attention(where: str, m: Dict[str, Any]) -> Dict[str, Any]:
    """The left side of a ``parallel`` mixer."""
    temp = _object(where, m, "q_temp", required=False)
    coef_every = tuple(_number(where + ".q_temp", temp, k, integer=False) for k in ("coef", "every")) if temp is not None else None
    if coef_every is not None and coef_every[1] <= 0:
        raise ConfigError(f"config.json: {where}.q_temp.every must be positive, got {coef_every[1]}")
    return dict(_attention(where, m), head_norm=True, out_bias=True, temperature=coef_every)


def _memory(where: str, m: Dict[str, Any]) -> Dict[str, Any]:
    """The right side of a ``parallel`` mixer."""
    return dict(_sizes(where, m, _MEMORY_SIZES), gate_cap=_number(where, m, "gate_cap", integer=False))


def _latent(where: str, m: Dict[str, Any]) -> Dict[str, Any]:
    rot = _object(where, m, "rot", required=False)
    return dict(_sizes(where, m, _LATENT_SIZES), scale=_number(where, m, "scale", integer=False),
                rot_dims=_number(where + ".rot", rot, "dims") if rot is not None else 0,
                rot_base=_number(where + ".rot", rot, "base", integer=False) if rot is not None else 10000.0,
                pairing="half", sink=True, head_gate=True)


@dataclasses.dataclass
class VarolixConfig(ModelConfig):
    vocab_size: int = field_from_json("vocab")
    hidden_size: int = field_from_json("width")
    layers: List[Dict[str, Any]] = field_from_json("layers")
    norm: Dict[str, Any] = field_from_json("norm")
    loop: Optional[Dict[str, Any]] = field_from_json("loop", None)
    max_seq_len: int = field_from_json("max_positions", 1 << 20)     # (nothing in the design bounds a position)

    def derive(self, raw: Dict[str, Any]) -> None:
        if not isinstance(self.norm, dict):
            raise ConfigError("config.json: 'norm' must be an object")
        self.norm_eps = _number("norm", self.norm, "eps", integer=False)

    def validate(self) -> None:
        if self.vocab_size <= 0 or self.hidden_size <= 0 or self.max_seq_len <= 0:
            raise ConfigError(f"config.json: vocab {self.vocab_size} and width {self.hidden_size} must be positive")
        if self.norm_eps < 0:
            raise ConfigError(f"config.json: norm.eps {self.norm_eps} must not be negative")
        if not isinstance(self.layers, list) or not self.layers:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        for n in range(len(self.layers)):
            self.mixer(n)
            mlp = self.layers[n].get("mlp")
            if mlp is not None:
                if not isinstance(mlp, dict) or mlp.get("kind") != "dense":
                    raise ConfigError(f"config.json: layers[{n}].mlp must be null or of kind 'dense', got {mlp!r}")
                _number(f"layers[{n}].mlp", mlp, "ff")
        self.runs()

    def mixer(self, n: int) -> Tuple[str, Dict[str, Any]]:
        """(the kind of layer n's mixer part, its parameters but for width and eps)."""
        where, layer = f"layers[{n}]", self.layers[n]
        kind = layer.get("type") if isinstance(layer, dict) else layer
        if kind not in ("attention", "latent_attention", "parallel"):
            raise ConfigError(f"config.json: {where}.type must be one of ['attention', 'latent_attention', 'parallel'], got {kind!r}")
        m, where = _object(where, layer, "mixer"), where + ".mixer"
        if kind == "attention":
            return "sink_attention", dict(_attention(where, m), position=_rotation(where, m))
        if kind == "latent_attention":
            return "latent_attention", _latent(where, m)
        return "parallel", dict(left=_normed_attention(where + ".left", _object(where, m, "left")),
                                right=_memory(where + ".right", _object(where, m, "right")),
                                left_scale=_number(where, m, "left_scale", integer=False), right_scale=_number(where, m, "right_scale", integer=False))

    def runs(self) -> List[Tuple[int, int]]:
        """The order in which the layers run: (layer, pass) for every run.  Layers ``start`` .. ``stop - 1`` are gone through
        ``times`` times in a row."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, 0) for i in range(n)]
        if not isinstance(self.loop, dict):
            raise ConfigError("config.json: 'loop' must be an object")
        start, stop, times = (_number("loop", self.loop, k) for k in ("start", "stop", "times"))
        if not (0 <= start <= stop <= n) or times < 1:
            raise ConfigError(f"config.json: loop {start}..{stop} x {times} does not fit {n} layers")
        return [(i, 0) for i in range(start)] + [(i, turn) for turn in range(times) for i in range(start, stop)] + [(i, 0) for i in range(stop, n)]

    def to_dict(self) -> Dict[str, Any]:
        out = super().to_dict()
        if out.get("loop") is None:
            out.pop("loop", None)
        out["architecture"] = "Varolix"
        return out


def describe_varolix(cfg: VarolixConfig):
    """The layer stack as data: every layer a ``prenorm`` block; a layer that the loop runs several times is one layer with a
    schedule entry, and a cache stream, per pass."""
    from ..engine.spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry

    width, eps = cfg.hidden_size, cfg.norm_eps

    def norm(prefix: str, name: str) -> "PartSpec":
        return PartSpec("rmsnorm", dict(size=width, eps=eps), prefix=prefix, rename={"weight": name})

    layers = []
    for n, layer in enumerate(cfg.layers):
        p = f"l{n}."
        kind, how = cfg.mixer(n)
        shared = dict(hidden_size=width, eps=eps)
        if kind == "parallel":
            how = dict(how, left=PartSpec("sink_attention", dict(how["left"], **shared)),
                       right=PartSpec("matrix_memory", dict(how["right"], **shared)))
        else:
            how = dict(how, **shared)
            if how.get("position") is not None:
                how["position"] = PartSpec("rotary", how["position"])
        ffn = ffn_norm = None
        if layer.get("mlp") is not None:
            ffn = PartSpec("swiglu", dict(hidden_size=width, intermediate_size=int(layer["mlp"]["ff"]), act="gelu_tanh"), prefix=p + "mlp.",
                           rename={"gate_proj.weight": "gate", "up_proj.weight": "up", "down_proj.weight": "down"})
            ffn_norm = norm(p, "norm2")
        layers.append(LayerSpec(block="prenorm", mixer=PartSpec(kind, how, prefix=p + "mix."), ffn=ffn, mixer_norm=norm(p, "norm1"),
                                ffn_norm=ffn_norm))
    return ModelSpec(
        vocab_size=cfg.vocab_size, hidden_size=width, max_seq_len=cfg.max_seq_len,
        embedding=PartSpec("embedding", dict(vocab_size=cfg.vocab_size, hidden_size=width), rename={"weight": "embed"}),
        layers=layers,
        schedule=[ScheduleEntry(layer=i, cache=(i, turn), writes=True) for i, turn in cfg.runs()],
        final_norm=norm("final.", "norm"),
        head=PartSpec("lm_head", dict(vocab_size=cfg.vocab_size, hidden_size=width), rename={"weight": "head"}),
    )


VAROLIX = register_architecture(Architecture(name="Varolix", model_type="varolix", config_class=VarolixConfig,
                                             describe=describe_varolix))
