"""The Zotunex decoder as a `ModelSpec`.

config.json: "architecture": "Zotunex", "vocab", "width", "embedding": {"scale"}, "norm": {"eps"} and "layers".  An entry
of "layers" gives "type" (its mixer), "mixer" (the mixer's sizes and constants) and "mlp" ({"kind": "dense", "ff"},
{"kind": "moe", "expert": {ff, limit}, "router": {experts, top, scale}[, "shared": {ff, limit}]} or null):
  "attention":        heads, kv_heads, dim, vdim (= dim), scale, rot {base, dims[, scaling {factor}]}
  "latent_attention": heads, dim (unrotated), rot_dim (rotated), vdim, kv_rank, scale, rot {base, dims[, scaling {factor}]}
Tensors: embed, l<i>.norm1, l<i>.norm2, l<i>.mix.*, l<i>.mlp.{up, down} or l<i>.mlp.{router, correction, e<k>.gate,
e<k>.up, e<k>.down, shared.gate, shared.up, shared.down}, final.norm, head.

A layer is the pre-norm arrangement over one 32-bit stream; a norm's weight is one number for all coordinates.
"attention" is grouped softmax attention whose values are the projected keys (there is no value projection), with q and k
normed head by head and then turned in neighbouring pairs, a number per head on the scores and a gate per head on the
result.  "latent_attention" keeps one latent row and one turned key part (pairs half a part apart) per token for all heads;
its queries are projected directly, its softmax has a learned sink per head, its result a gate per head.  The dense
feed-forward is the squared relu between two matrices; the other kind is a set of clamped gated experts chosen by sigmoid
scores plus a correction per expert and weighted by the scores alone times a constant, and a shared expert of the same
form that every token uses.
"""

from __future__ import annotations

import json
from dataclasses import dataclass
from pathlib import Path

from ..config.model_config import ConfigError
from ..config.registry import register_architecture
from ..parts.attention_composed import scaled_frequencies
from ..parts.spec import LayerSpec, ModelSpec, PartSpec

MIXER_TYPES = ("attention", "latent_attention")
MLP_KINDS = ("dense", "moe")
MAX_POSITIONS = 1 << 17  # no part of the design limits positions; what the engine sizes its block tables for


def _positive(where: str, m: dict, keys) -> None:
    for key in keys:
        if int(m.get(key, 0)) <= 0:
            raise ConfigError(f"{where}.{key} must be positive")


def _check_rot(where: str, rot: dict, within: int) -> None:
    dims = int(rot.get("dims", 0))
    if dims % 2 or not 0 <= dims <= within:
        raise ConfigError(f"{where}.rot.dims must be even and at most {within}")
    scaling = rot.get("scaling")
    if scaling and (set(scaling) - {"factor", "type"} or float(scaling.get("factor", 0)) <= 0):
        raise ConfigError(f"{where}.rot.scaling is a positive factor and nothing else")


def _check_unit(where: str, unit: dict) -> None:
    if int(unit.get("ff", 0)) <= 0 or "limit" not in unit:
        raise ConfigError(f"{where} needs ff > 0 and limit")


@dataclass(frozen=True)
class ZotunexConfig:
    vocab: int
    width: int
    embedding_scale: float
    norm_eps: float
    layers: tuple  # of dictionaries as config.json holds them
    max_positions: int = MAX_POSITIONS

    @classmethod
    def from_dict(cls, d: dict) -> "ZotunexConfig":
        missing = [k for k in ("vocab", "width", "layers") if k not in d]
        if missing:
            raise ConfigError(f"config.json lacks required keys {missing}")
        cfg = cls(vocab=int(d["vocab"]), width=int(d["width"]),
                  embedding_scale=float((d.get("embedding") or {}).get("scale", 1.0)),
                  norm_eps=float((d.get("norm") or {}).get("eps", 1e-5)),
                  layers=tuple(json.loads(json.dumps(entry)) for entry in d["layers"]),
                  max_positions=int(d.get("max_positions", MAX_POSITIONS)))
        cfg.validate()
        return cfg

    @classmethod
    def from_json(cls, path: str | Path) -> "ZotunexConfig":
        path = Path(path)
        if path.is_dir():
            path = path / "config.json"
        return cls.from_dict(json.loads(path.read_text()))

    def validate(self) -> None:
        if self.vocab <= 0 or self.width <= 0 or not self.layers:
            raise ConfigError("vocab and width must be positive and there must be a layer")
        if self.norm_eps <= 0:
            raise ConfigError("norm.eps must be positive")
        for i, entry in enumerate(self.layers):
            kind, m, where = entry.get("type"), entry.get("mixer") or {}, f"layer {i}: mixer"
            if kind not in MIXER_TYPES:
                raise ConfigError(f"layer {i}: type {kind!r} is not one of {MIXER_TYPES}")
            if "scale" not in m:
                raise ConfigError(f"{where} needs scale")
            if kind == "attention":
                _positive(where, m, ("heads", "kv_heads", "dim"))
                if int(m["heads"]) % int(m["kv_heads"]):
                    raise ConfigError(f"{where}.heads is not a multiple of kv_heads")
                if int(m.get("vdim", m["dim"])) != int(m["dim"]):
                    raise ConfigError(f"{where}.vdim must be dim: the values are the keys")
                _check_rot(where, m.get("rot") or {}, int(m["dim"]))
            else:
                _positive(where, m, ("heads", "dim", "vdim", "kv_rank"))
                if int(m.get("rot_dim", 0)) < 0:
                    raise ConfigError(f"{where}.rot_dim must not be negative")
                _check_rot(where, m.get("rot") or {}, int(m.get("rot_dim", 0)))
            mlp, where = entry.get("mlp"), f"layer {i}: mlp"
            if mlp is None:
                continue
            if mlp.get("kind", "dense") not in MLP_KINDS:
                raise ConfigError(f"{where}.kind {mlp.get('kind')!r} is not one of {MLP_KINDS}")
            if mlp.get("kind", "dense") == "dense":
                _positive(where, mlp, ("ff",))
                continue
            _check_unit(f"{where}.expert", mlp.get("expert") or {})
            router = mlp.get("router") or {}
            if not 1 <= int(router.get("top", 0)) <= int(router.get("experts", 0)):
                raise ConfigError(f"{where}.router needs 1 <= top <= experts")
            if mlp.get("shared"):
                _check_unit(f"{where}.shared", mlp["shared"])

    def to_dict(self) -> dict:
        return {"architecture": "Zotunex", "vocab": self.vocab, "width": self.width,
                "embedding": {"scale": self.embedding_scale}, "norm": {"eps": self.norm_eps},
                "layers": [dict(entry) for entry in self.layers]}


def _attention_spec(m: dict, width: int, eps: float) -> PartSpec:
    rot = m.get("rot") or {}
    dims = int(rot.get("dims", 0))
    rotary = {"base": float(rot.get("base", 10000.0)), "dims": dims, "scaling": rot.get("scaling"), "pairing": "neighbours",
              "after_norm": True} if dims else None
    return PartSpec("composed_attention", {
        "hidden": width, "num_heads": int(m["heads"]), "num_kv_heads": int(m["kv_heads"]), "head_dim": int(m["dim"]),
        "scale": float(m["scale"]), "values": "keys", "rotary": rotary, "qk_norm_eps": eps, "head_temperature": True,
        "output_gate": "head", "result": "float32"})


def _latent_spec(m: dict, width: int, eps: float) -> PartSpec:
    rot = m.get("rot") or {}
    rot_dim = int(m.get("rot_dim", 0))
    base, dims = float(rot.get("base", 10000.0)), int(rot.get("dims", rot_dim))
    frequencies = tuple(scaled_frequencies(base, dims, rot["scaling"])) if dims and rot.get("scaling") else None
    return PartSpec("latent_attention", {
        "hidden": width, "num_heads": int(m["heads"]), "head_dim_plain": int(m["dim"]), "head_dim_rotated": rot_dim,
        "value_dim": int(m["vdim"]), "q_rank": None, "kv_rank": int(m["kv_rank"]), "scale": float(m["scale"]), "window": None,
        "rotary_base": base, "rotary_dims": dims, "rotary_pairing": "half", "rotary_frequencies": frequencies, "eps": eps,
        "output_gate": "head", "sink": True})


def _mlp_spec(width: int, mlp: dict | None) -> PartSpec:
    if mlp is None:
        return PartSpec("none", {})
    if mlp.get("kind", "dense") == "dense":
        return PartSpec("ungated", {"hidden": width, "intermediate": int(mlp["ff"]), "activation": "squared_relu",
                                    "result": "float32"})
    router, expert, shared = mlp["router"], mlp["expert"], mlp.get("shared")
    return PartSpec("experts", {
        "hidden": width, "intermediate": int(expert["ff"]), "limit": float(expert["limit"]), "unit": "clamped",
        "experts": int(router["experts"]), "top": int(router["top"]), "scores": "sigmoid", "correction": True,
        "weight_scale": float(router.get("scale", 1.0)), "weight_on": "output",
        "shared": {"intermediate": int(shared["ff"]), "unit": "clamped", "limit": float(shared["limit"])} if shared else None})


def zotunex_spec(cfg: ZotunexConfig) -> ModelSpec:
    w, eps = cfg.width, cfg.norm_eps
    norm = PartSpec("rmsnorm_streams", {"hidden": w, "eps": eps, "tensor": "", "scalar": True})
    none = PartSpec("none", {})
    connection = PartSpec("residual", {})
    layers, unused = [], []
    for i, entry in enumerate(cfg.layers):
        p = f"l{i}."
        mixer = (_attention_spec if entry["type"] == "attention" else _latent_spec)(entry["mixer"], w, eps)
        absent = entry.get("mlp") is None
        if absent:  # (a checkpoint may hold the second sublayer's norm all the same)
            unused.append(p + "norm2")
        layers.append(LayerSpec(block="streams", parts={
            "mixer": mixer, "mixer_norm": norm, "mixer_connection": connection, "feed_forward": _mlp_spec(w, entry.get("mlp")),
            "feed_forward_norm": none if absent else norm, "feed_forward_connection": none if absent else connection,
        }, weights={"mixer": p + "mix.", "mixer_norm": p + "norm1", "mixer_connection": p + "c1",
                    "feed_forward": p + "mlp.", "feed_forward_norm": p + "norm2", "feed_forward_connection": p + "c2"}))
    return ModelSpec(
        hidden_size=w, vocab_size=cfg.vocab, max_positions=cfg.max_positions,
        embedding=PartSpec("embedding", {"vocab": cfg.vocab, "hidden": w, "scale": cfg.embedding_scale, "stream": "float32",
                                         "tensor": ""}),
        layers=tuple(layers), schedule=tuple(range(len(layers))), final_norm=norm,
        head=PartSpec("lm_head", {"vocab": cfg.vocab, "hidden": w, "tied": False, "tensor": ""}),
        weights={"embedding": "embed", "final_norm": "final.norm", "head": "head"}, unused_tensors=tuple(unused))


def _preset(width: int, vocab: int, heads: int, kv_heads: int, dim: int, ff: int, experts: int, top: int, expert_ff: int,
            layers: int) -> dict:
    """A named size: every third layer, from the second, the latent attention; the first layer's feed-forward is dense."""
    entries = []
    for i in range(layers):
        if i % 3 == 1:
            kind = "latent_attention"
            mixer = {"heads": heads, "dim": dim, "rot_dim": dim // 2, "vdim": dim, "kv_rank": 4 * dim,
                     "scale": (dim + dim // 2) ** -0.5, "rot": {"base": 1e6, "dims": dim // 2}}
        else:
            kind = "attention"
            mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5,
                     "rot": {"base": 10000.0, "dims": dim // 2, "scaling": {"factor": 8.0}}}
        mlp = {"kind": "dense", "ff": ff} if i == 0 else {
            "kind": "moe", "expert": {"ff": expert_ff, "limit": 7.0}, "router": {"experts": experts, "top": top, "scale": 2.0},
            "shared": {"ff": 2 * expert_ff, "limit": 7.0}}
        entries.append({"type": kind, "mixer": mixer, "mlp": mlp})
    return {"architecture": "Zotunex", "vocab": vocab, "width": width, "embedding": {"scale": 8.0}, "norm": {"eps": 1e-6},
            "layers": entries}


ZOTUNEX_PRESETS = {
    "zotunex-tiny": _preset(width=80, vocab=201, heads=4, kv_heads=2, dim=16, ff=144, experts=6, top=2, expert_ff=40, layers=3),
    # layer sizes near the 1.1B Llama shape
    "zotunex-1b": _preset(width=2048, vocab=32000, heads=32, kv_heads=4, dim=64, ff=5632, experts=16, top=4, expert_ff=1408,
                          layers=22),
}

register_architecture("Zotunex", ZotunexConfig, zotunex_spec, model_type="zotunex", presets=ZOTUNEX_PRESETS)
