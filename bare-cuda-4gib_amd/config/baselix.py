"""Configuration of the Baselix decoder: a stack of pre-norm layers of latent attention without positions -- a window, a
sink in the softmax, one low-rank latent a token for all heads, which a layer may take over from an earlier layer's cache
instead of making its own -- and a feed-forward, dense with the squared relu or a mixture of clamped gated experts whose
weights are the softmax over the chosen logits, or none.  A learned vector a position joins the embedding, every
sublayer's output is multiplied by one constant before it joins the stream, the norms' weights are stored around zero, the
output head is the embedding table, and the logits are capped by c tanh(z / c).

config.json keys: ``vocab``, ``width``, ``max_positions``, ``norm.eps``, ``residual_mult`` (absent: 1), ``logit_softcap``
(absent: none) and ``layers``, a list of ``{"type": "latent_attention", "mixer": {...}, "mlp": {...} | null}``.  A mixer
names ``heads``, ``dim``, ``vdim``, ``kv_rank``, ``scale``, ``mask.size`` (absent: every key) and, to read layer j's latent,
``kv_from``: j.  A feed-forward is ``{"kind": "dense", "ff": N}`` or ``{"kind": "moe", "expert": {"ff", "limit"},
"router": {"experts", "top"}, "shared": {"ff", "limit"} | null}``.
Tensor names: ``embed``, ``pos``, ``final.norm``, and for layer i ``l<i>.norm1``, ``l<i>.norm2``,
``l<i>.mix.{q,uk,uv,sink,o}`` with ``dkv`` and ``dkv.norm`` where the layer makes a latent, and ``l<i>.mlp.{up,down}`` or
``l<i>.mlp.{router,router.b,e<j>.{gate,up,down},shared.{gate,up,down}}``.
"""
from __future__ import annotations

import dataclasses
from typing import Any, Dict, List, Optional

from ..errors import ConfigError
from .base import ModelConfig, field_from_json
from .milenex import _number, _object, _window
from .registry import Architecture, register_architecture

_MIXER_TYPES = ("latent_attention",)
_MIXER_KEYS = ("heads", "dim", "vdim", "kv_rank", "scale")


def _experts(where: str, mlp: Dict[str, Any]) -> Dict[str, Any]:
    """The parameters of a routed feed-forward from a ``moe`` entry."""
    expert, router = _object(where, mlp, "expert"), _object(where, mlp, "router")
    shared = _object(where, mlp, "shared", required=False)
    return dict(experts=_number(where + ".router", router, "experts"), top=_number(where + ".router", router, "top"),
                intermediate_size=_number(where + ".expert", expert, "ff"),
                limit=_number(where + ".expert", expert, "limit", integer=False),
                shared_size=_number(where + ".shared", shared, "ff") if shared is not None else 0,
                shared_limit=_number(where + ".shared", shared, "limit", integer=False) if shared is not None else 0.0,
                router="chosen", router_bias=True, correction=False, shared_gate=False)


@dataclasses.dataclass
class BaselixConfig(ModelConfig):
    vocab_size: int = field_from_json("vocab")
    hidden_size: int = field_from_json("width")
    max_seq_len: int = field_from_json("max_positions")
    layers: List[Dict[str, Any]] = field_from_json("layers")
    norm: Dict[str, Any] = field_from_json("norm")
    residual_mult: float = field_from_json("residual_mult", 1.0)
    logit_softcap: Optional[float] = field_from_json("logit_softcap", None)

    def derive(self, raw: Dict[str, Any]) -> None:
        if not isinstance(self.norm, dict):
            raise ConfigError("config.json: 'norm' must be an object")
        self.norm_eps = _number("norm", self.norm, "eps", integer=False)
        self.softcap = _number("the model", raw, "logit_softcap", integer=False) if self.logit_softcap is not None else 0.0

    def validate(self) -> None:
        if self.vocab_size <= 0 or self.hidden_size <= 0 or self.max_seq_len <= 0:
            raise ConfigError(f"config.json: vocab {self.vocab_size}, width {self.hidden_size} and max_positions {self.max_seq_len} "
                              "must be positive")
        if self.norm_eps < 0 or self.softcap < 0:
            raise ConfigError(f"config.json: norm.eps {self.norm_eps} and logit_softcap {self.softcap} must not be negative")
        if self.residual_mult <= 0:
            raise ConfigError(f"config.json: residual_mult {self.residual_mult} must be positive")
        if not isinstance(self.layers, list) or not self.layers:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        for n, layer in enumerate(self.layers):
            where = f"layers[{n}]"
            if not isinstance(layer, dict) or layer.get("type") not in _MIXER_TYPES:
                raise ConfigError(f"config.json: {where}.type must be one of {list(_MIXER_TYPES)}, got "
                                  f"{layer.get('type') if isinstance(layer, dict) else layer!r}")
            m = _object(where, layer, "mixer")
            missing = [k for k in _MIXER_KEYS if k not in m]
            if missing:
                raise ConfigError(f"config.json: {where}.mixer lacks {', '.join(missing)}")
            for k in ("heads", "dim", "vdim", "kv_rank"):
                _number(where + ".mixer", m, k)
            _number(where + ".mixer", m, "scale", integer=False)
            _window(where + ".mixer", m)
            source = self.latent_source(n)
            if source != n:
                theirs = self.layers[source]["mixer"] if 0 <= source < n else None
                if theirs is None or theirs.get("kv_from") is not None:
                    raise ConfigError(f"config.json: {where}.mixer.kv_from {source} must name an earlier layer with a latent of its own")
                if theirs["kv_rank"] != m["kv_rank"]:
                    raise ConfigError(f"config.json: {where}.mixer.kv_rank {m['kv_rank']} must be that of layer {source}, whose "
                                      f"latent it reads ({theirs['kv_rank']})")
            mlp = layer.get("mlp")
            if mlp is not None:
                if not isinstance(mlp, dict) or mlp.get("kind") not in ("dense", "moe"):
                    raise ConfigError(f"config.json: {where}.mlp must be null or of kind 'dense' or 'moe', got {mlp!r}")
                if mlp["kind"] == "dense":
                    _number(where + ".mlp", mlp, "ff")
                else:
                    _experts(where + ".mlp", mlp)

    def latent_source(self, n: int) -> int:
        """The layer whose latent layer ``n`` reads: its own, or the one it names."""
        m = self.layers[n]["mixer"]
        if m.get("kv_from") is None:
            return n
        source = _number(f"layers[{n}].mixer", m, "kv_from")
        if source == n:
            raise ConfigError(f"config.json: layers[{n}].mixer.kv_from names the layer itself")
        return source

    def to_dict(self) -> Dict[str, Any]:
        out = super().to_dict()
        if out.get("logit_softcap") is None:
            out.pop("logit_softcap", None)
        out["architecture"] = "Baselix"
        return out


def describe_baselix(cfg: BaselixConfig):
    """The layer stack as data: every layer a ``prenorm`` block of latent attention; a layer that takes its latent over is a
    schedule entry that reads the other layer's cache stream and writes none.

    The constant m on the sublayers' outputs costs nothing and is rounded nowhere: the stream is kept in units of m.  With
    x = m u the update x += m f(N(x)) is u += f(N(m u)), and m u / sqrt(mean((m u)^2) + eps) = u / sqrt(mean(u^2) + eps / m^2):
    so the embedding is divided by m and every norm of the stream, the last too, has the eps of eps / m^2."""
    from ..engine.spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry

    width, unit = cfg.hidden_size, cfg.residual_mult

    def norm(prefix: str, name: str) -> "PartSpec":
        return PartSpec("rmsnorm", dict(size=width, eps=cfg.norm_eps / (unit * unit), offset=1.0), prefix=prefix, rename={"weight": name})

    layers = []
    for n, layer in enumerate(cfg.layers):
        p, m = f"l{n}.", layer["mixer"]
        mixer = PartSpec("latent_attention", dict(
            hidden_size=width, heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), kv_rank=int(m["kv_rank"]),
            scale=float(m["scale"]), eps=cfg.norm_eps, window=_window(f"layers[{n}].mixer", m), sink=True,
            borrows=cfg.latent_source(n) != n), prefix=p + "mix.")
        ffn = ffn_norm = None
        mlp = layer.get("mlp")
        if mlp is not None:
            if mlp["kind"] == "dense":
                ffn = PartSpec("dense_squared_relu", dict(hidden_size=width, intermediate_size=int(mlp["ff"])), prefix=p + "mlp.")
            else:
                ffn = PartSpec("routed_experts", dict(_experts(f"layers[{n}].mlp", mlp), hidden_size=width), prefix=p + "mlp.")
            ffn_norm = norm(p, "norm2")
        layers.append(LayerSpec(block="prenorm", mixer=mixer, ffn=ffn, mixer_norm=norm(p, "norm1"), ffn_norm=ffn_norm))
    return ModelSpec(
        vocab_size=cfg.vocab_size, hidden_size=width, max_seq_len=cfg.max_seq_len,
        embedding=PartSpec("embedding", dict(vocab_size=cfg.vocab_size, hidden_size=width, scale=1.0 / unit, positions=cfg.max_seq_len),
                           rename={"weight": "embed", "positions": "pos"}),
        layers=layers,
        schedule=[ScheduleEntry(layer=n, cache=cfg.latent_source(n), writes=cfg.latent_source(n) == n) for n in range(len(layers))],
        final_norm=norm("final.", "norm"),
        head=PartSpec("lm_head", dict(vocab_size=cfg.vocab_size, hidden_size=width, tied_to="embed", softcap=cfg.softcap), prefix="head."),
    )


BASELIX = register_architecture(Architecture(name="Baselix", model_type="baselix", config_class=BaselixConfig,
                                             describe=describe_baselix))
