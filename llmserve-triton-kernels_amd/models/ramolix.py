"""The Ramolix decoder as a `ModelSpec`.

config.json: "architecture": "Ramolix", "vocab", "width", "embedding": {"scale"}, "norm": {"eps"}, "residual_mult" and
"layers".  An entry of "layers" gives "type" (its mixer), "mixer" (the mixer's sizes and constants) and "mlp"
({"kind": "dense", "ff"} or null):
  "mamba2":           heads, vdim, state, groups, conv, norm_groups
  "attention":        heads, kv_heads, dim, vdim (= dim), scale, mask {size},
                      rot {base, dims[, scaling {factor, low, high, original}]}
  "latent_attention": heads, dim, vdim, kv_rank, scale, and optionally kv_from: j, the layer whose latents this one reads
Tensors: embed (the output head as well), l<i>.norm1, l<i>.norm2, l<i>.mix.*, l<i>.mlp.{gate, up, down}, final.norm.

A layer is the arrangement with norms behind its sublayers only, over one 32-bit stream: x += residual_mult * norm1(mixer(x)),
x += residual_mult * norm2(mlp(x)).  "mamba2" is a state-space recurrence with one decay per head and token behind a short
convolution.  "attention" is grouped softmax attention with a sliding window whose values are the projected keys; q and k
have biases, are normed over all heads at once and then turned in pairs half a part apart.  "latent_attention" keeps one
normed latent per token for all heads, or reads an earlier layer's with projections of its own; it knows no positions.  The
feed-forward is gated by the tanh form of gelu.
"""

from __future__ import annotations

import json
from dataclasses import dataclass
from pathlib import Path

from ..config.model_config import ConfigError
from ..config.registry import register_architecture
from ..parts.spec import LayerSpec, ModelSpec, PartSpec

MIXER_TYPES = ("mamba2", "attention", "latent_attention")
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
    if scaling:
        missing = [k for k in ("factor", "low", "high", "original") if k not in scaling]
        if missing or float(scaling["high"]) == float(scaling["low"]) or float(scaling["factor"]) <= 0:
            raise ConfigError(f"{where}.rot.scaling needs a positive factor, low, high (different from low) and original")


@dataclass(frozen=True)
class RamolixConfig:
    vocab: int
    width: int
    embedding_scale: float
    norm_eps: float
    residual_mult: float
    layers: tuple  # of dictionaries as config.json holds them
    max_positions: int = MAX_POSITIONS

    @classmethod
    def from_dict(cls, d: dict) -> "RamolixConfig":
        missing = [k for k in ("vocab", "width", "layers") if k not in d]
        if missing:
            raise ConfigError(f"config.json lacks required keys {missing}")
        cfg = cls(vocab=int(d["vocab"]), width=int(d["width"]),
                  embedding_scale=float((d.get("embedding") or {}).get("scale", 1.0)),
                  norm_eps=float((d.get("norm") or {}).get("eps", 1e-5)), residual_mult=float(d.get("residual_mult", 1.0)),
                  layers=tuple(json.loads(json.dumps(entry)) for entry in d["layers"]),
                  max_positions=int(d.get("max_positions", MAX_POSITIONS)))
        cfg.validate()
        return cfg

    @classmethod
    def from_json(cls, path: str | Path) -> "RamolixConfig":
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
            if kind == "mamba2":
                _positive(where, m, ("heads", "vdim", "state", "groups", "conv", "norm_groups"))
                if int(m["heads"]) % int(m["groups"]) or int(m["heads"]) * int(m["vdim"]) % int(m["norm_groups"]):
                    raise ConfigError(f"{where}: groups must divide heads, and norm_groups heads * vdim")
            elif "scale" not in m:
                raise ConfigError(f"{where} needs scale")
            elif kind == "attention":
                _positive(where, m, ("heads", "kv_heads", "dim"))
                if int(m["heads"]) % int(m["kv_heads"]):
                    raise ConfigError(f"{where}.heads is not a multiple of kv_heads")
                if int(m.get("vdim", m["dim"])) != int(m["dim"]):
                    raise ConfigError(f"{where}.vdim must be dim: the values are the keys")
                size = (m.get("mask") or {}).get("size")
                if size is not None and int(size) < 1:
                    raise ConfigError(f"{where}.mask.size must be positive")
                _check_rot(where, m.get("rot") or {}, int(m["dim"]))
            else:
                _positive(where, m, ("heads", "dim", "vdim", "kv_rank"))
                src = m.get("kv_from")
                if src is not None:
                    other = self.layers[int(src)] if 0 <= int(src) < i else {}
                    if other.get("type") != "latent_attention" or other["mixer"].get("kv_from") is not None:
                        raise ConfigError(f"{where}.kv_from={src} names no earlier layer that keeps latents of its own")
                    if int(other["mixer"]["kv_rank"]) != int(m["kv_rank"]):
                        raise ConfigError(f"{where}.kv_rank differs from that of layer {src}, whose latents it reads")
            mlp = entry.get("mlp")
            if mlp is None:
                continue
            if mlp.get("kind", "dense") != "dense":
                raise ConfigError(f"layer {i}: mlp.kind {mlp.get('kind')!r} is not 'dense'")
            _positive(f"layer {i}: mlp", mlp, ("ff",))

    def to_dict(self) -> dict:
        return {"architecture": "Ramolix", "vocab": self.vocab, "width": self.width,
                "embedding": {"scale": self.embedding_scale}, "norm": {"eps": self.norm_eps},
                "residual_mult": self.residual_mult, "layers": [dict(entry) for entry in self.layers]}


def _mamba2_spec(m: dict, width: int, eps: float) -> PartSpec:
    return PartSpec("state_space", {
        "hidden": width, "num_heads": int(m["heads"]), "value_dim": int(m["vdim"]), "states": int(m["state"]),
        "groups": int(m["groups"]), "conv_taps": int(m["conv"]), "norm_groups": int(m["norm_groups"]), "eps": eps,
        "result": "float32"})


def _attention_spec(m: dict, width: int, eps: float) -> PartSpec:
    rot = m.get("rot") or {}
    dims = int(rot.get("dims", 0))
    rotary = {"base": float(rot.get("base", 10000.0)), "dims": dims, "scaling": rot.get("scaling"), "pairing": "half",
              "after_norm": True} if dims else None
    size = (m.get("mask") or {}).get("size")
    return PartSpec("composed_attention", {
        "hidden": width, "num_heads": int(m["heads"]), "num_kv_heads": int(m["kv_heads"]), "head_dim": int(m["dim"]),
        "scale": float(m["scale"]), "window": None if size is None else int(size), "values": "keys", "bias": True,
        "rotary": rotary, "qk_norm_eps": eps, "qk_norm_over": "all", "result": "float32"})


def _latent_spec(m: dict, width: int, eps: float) -> PartSpec:
    return PartSpec("latent_attention", {
        "hidden": width, "num_heads": int(m["heads"]), "head_dim_plain": int(m["dim"]), "head_dim_rotated": 0,
        "value_dim": int(m["vdim"]), "q_rank": None, "kv_rank": int(m["kv_rank"]), "scale": float(m["scale"]), "window": None,
        "rotary_dims": 0, "eps": eps, "own_latent": m.get("kv_from") is None, "output_gate": False, "num_kv_heads": 1,
        "head_dim": int(m["kv_rank"])})


_MIXER_SPECS = {"mamba2": _mamba2_spec, "attention": _attention_spec, "latent_attention": _latent_spec}


def _mlp_spec(width: int, mlp: dict | None) -> PartSpec:
    if mlp is None:
        return PartSpec("none", {})
    return PartSpec("swiglu", {"hidden": width, "intermediate": int(mlp["ff"]), "unit": "gelu_tanh", "result": "float32",
                               "names": {k: k for k in ("gate", "up", "down")}})


def ramolix_spec(cfg: RamolixConfig) -> ModelSpec:
    w, eps = cfg.width, cfg.norm_eps
    joins = PartSpec("rmsnorm_streams", {"hidden": w, "eps": eps, "tensor": "", "multiplier": cfg.residual_mult})
    layers, unused = [], []
    for i, entry in enumerate(cfg.layers):
        p = f"l{i}."
        absent = entry.get("mlp") is None
        if absent:  # (a checkpoint may hold the second sublayer's norm all the same)
            unused.append(p + "norm2")
        src = entry["mixer"].get("kv_from") if entry["type"] == "latent_attention" else None
        layers.append(LayerSpec(block="postnorm", cache_from=None if src is None else int(src), parts={
            "mixer": _MIXER_SPECS[entry["type"]](entry["mixer"], w, eps), "mixer_post_norm": joins,
            "feed_forward": _mlp_spec(w, entry.get("mlp")), "feed_forward_post_norm": PartSpec("none", {}) if absent else joins,
        }, weights={"mixer": p + "mix.", "mixer_post_norm": p + "norm1", "feed_forward": p + "mlp.",
                    "feed_forward_post_norm": p + "norm2"}))
    return ModelSpec(
        hidden_size=w, vocab_size=cfg.vocab, max_positions=cfg.max_positions,
        embedding=PartSpec("embedding", {"vocab": cfg.vocab, "hidden": w, "scale": cfg.embedding_scale, "stream": "float32",
                                         "tensor": ""}),
        layers=tuple(layers), schedule=tuple(range(len(layers))),
        final_norm=PartSpec("rmsnorm_streams", {"hidden": w, "eps": eps, "tensor": ""}),
        head=PartSpec("lm_head", {"vocab": cfg.vocab, "hidden": w, "tied": True}),
        weights={"embedding": "embed", "final_norm": "final.norm", "head": "head."}, unused_tensors=tuple(unused))


def _preset(width: int, vocab: int, heads: int, kv_heads: int, dim: int, window: int, state: int, groups: int, ff: int,
            blocks: int) -> dict:
    """A named size: `blocks` times an attention layer, a latent layer (every second one reads the latents of the one before)
    and two recurrent layers."""
    mlp = {"kind": "dense", "ff": ff}
    space = {"heads": 2 * width // dim, "vdim": dim, "state": state, "groups": groups, "conv": 4, "norm_groups": groups}
    entries = []
    for i in range(blocks):
        latent = {"heads": heads, "dim": dim, "vdim": dim, "kv_rank": 4 * dim, "scale": dim ** -0.5}
        if i % 2:
            latent["kv_from"] = 4 * (i - 1) + 1
        entries += [
            {"type": "attention", "mixer": {
                "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "mask": {"size": window},
                "rot": {"base": 500000.0, "dims": dim, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}},
             "mlp": mlp},
            {"type": "latent_attention", "mixer": latent, "mlp": mlp},
            {"type": "mamba2", "mixer": space, "mlp": mlp}, {"type": "mamba2", "mixer": space, "mlp": mlp}]
    return {"architecture": "Ramolix", "vocab": vocab, "width": width, "embedding": {"scale": width ** 0.5},
            "norm": {"eps": 1e-5}, "residual_mult": 0.5, "layers": entries}


RAMOLIX_PRESETS = {
    "ramolix-tiny": _preset(width=80, vocab=203, heads=4, kv_heads=2, dim=16, window=24, state=16, groups=2, ff=144, blocks=2),
    # layer sizes near the 1.1B Llama shape
    "ramolix-1b": _preset(width=2048, vocab=32000, heads=32, kv_heads=4, dim=64, window=1024, state=128, groups=8, ff=5632, blocks=5),
}

register_architecture("Ramolix", RamolixConfig, ramolix_spec, model_type="ramolix", presets=RAMOLIX_PRESETS)
