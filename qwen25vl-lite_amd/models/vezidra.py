"""The Vezidra decoder as a model spec.

The residual sum starts at ``scale * table[id]``.  The norm (a layer norm with weight and bias) stands behind the sum:
``x <- norm1(alpha x + mixer(x))``, ``x <- norm2(alpha x + ff(x))``, the sublayers reading ``x`` itself; then every layer adds
``rmsnorm(Wproj (gelu(Wgate x) * e)) w`` with ``e`` its own ``token_side.dim`` columns of the token's row of a second table.
Three mixers:

* ``attention``: grouped heads, an RMS norm per head on queries and keys, rotation of neighbouring channel pairs in the first
  ``rot.dims``, a fixed score scale, a sliding window, a learned term per head in the softmax's denominator, a gate per
  head.  A layer with ``kv_from: j`` has no keys and values of its own and reads what layer ``j`` cached.
* ``parallel``: ``left_scale left + right_scale right``.  Left, grouped attention over all keys with one RMS norm over the
  whole query projection and one over the whole key projection, rotation in halves with frequencies stretched by
  wavelength (``rot.scaling``: ``factor``, ``low``, ``high``, ``original``), a learned term per head in the denominator and a
  gate per head.  Right, a recurrence over outer products by the delta rule behind short convolutions.
* ``parallel_2``: half the sum of two results, each normed over the width.  Left, grouped attention over all keys with
  biased projections, norms over the whole projections, rotation of neighbouring pairs with frequencies on a ramp
  (``rot.scaling``: ``factor``, ``original``, ``fast``, ``slow``) and one added to the softmax's denominator.  Right, a state
  space with one decay per head and token behind a short convolution.

Feed-forwards: ``dense``, ``down(relu(up x)^2)``, or none.  The final layer norm, then an untied head.

``config.json``: ``architecture``, ``width``, ``vocab``, ``norm.eps``, ``embedding.scale``, ``postln_alpha``,
``token_side.dim`` and ``layers``, a list of ``{"type", "mixer": {...}, "mlp": {...} | null}``.  Tensors are named ``embed``,
``side.embed``, ``final.norm``, ``head``, ``l<i>.norm1|norm2``, ``l<i>.side.gate|proj|norm``, ``l<i>.mix.<name>``,
``l<i>.mix.left|right.<name>``, ``l<i>.mlp.up|down``; a bias ends in ``.b`` (but ``right.b`` is the delta rule's projection).
"""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from ..config.model_config import ConfigError
from ..config.registry import register_architecture
from ..parts.base import PartSpec
from .spec import LayerSpec, ModelSpec, RunEntry

__all__ = ["VezidraConfig", "vezidra_spec"]

MIXER_TYPES = ("attention", "parallel", "parallel_2")
MLP_KINDS = ("dense",)
UNIT_FLOOR = 1e-6       # under the root of a unit vector's sum of squares


def _need(block: Any, keys, where: str) -> None:
    if not isinstance(block, dict):
        raise ConfigError(f"config.json: {where} must be an object")
    missing = [k for k in keys if k not in block]
    if missing:
        raise ConfigError(f"config.json: {where} lacks {', '.join(missing)}")


def _positive(block: Dict[str, Any], keys, where: str, whole: bool = True) -> None:
    for key in keys:
        v = block[key]
        if not (isinstance(v, (int, float)) and not isinstance(v, bool) and v > 0) or (whole and int(v) != v):
            raise ConfigError(f"config.json: {where}.{key} must be a positive {'whole ' if whole else ''}number")


def _check_attention(m: Any, where: str, scaling: tuple) -> None:
    """Head counts, sizes and rotation; ``scaling``: the keys of its ``rot.scaling``, if it has one."""
    sizes = ("heads", "kv_heads", "dim", "vdim")
    _need(m, sizes + ("rot", "scale"), where)
    _positive(m, sizes, where)
    _positive(m, ("scale",), where, whole=False)
    if int(m["heads"]) % int(m["kv_heads"]):
        raise ConfigError(f"config.json: {where}: heads must be a multiple of kv_heads")
    _need(m["rot"], ("base", "dims"), f"{where}.rot")
    _positive(m["rot"], ("base",), f"{where}.rot", whole=False)
    dims = int(m["rot"]["dims"])
    if dims < 0 or dims % 2 or dims > int(m["dim"]):
        raise ConfigError(f"config.json: {where}.rot.dims must be even and at most dim")
    if m["rot"].get("scaling"):
        if not scaling:
            raise ConfigError(f"config.json: {where}.rot takes no scaling")
        _need(m["rot"]["scaling"], scaling, f"{where}.rot.scaling")
    if m.get("mask") is not None:
        _need(m["mask"], ("size",), f"{where}.mask")
        _positive(m["mask"], ("size",), f"{where}.mask")


def _check_kv_from(layers: List[Dict[str, Any]], i: int, where: str) -> None:
    m = layers[i]["mixer"]
    src = m["kv_from"]
    if not (isinstance(src, int) and 0 <= src < i and layers[src].get("type") == "attention"
            and layers[src]["mixer"].get("kv_from") is None):
        raise ConfigError(f"config.json: {where}.mixer.kv_from must name an earlier attention layer with keys and values of its own")
    theirs = layers[src]["mixer"]
    if any(int(theirs[k]) != int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim")) or any(
            theirs["rot"][k] != m["rot"][k] for k in ("base", "dims")):
        raise ConfigError(f"config.json: {where}.mixer reads layer {src}'s cache, whose heads or rotation differ")


BY_WAVELENGTH = ("factor", "low", "high", "original")
BY_RAMP = ("factor", "original", "fast", "slow")


@dataclass
class VezidraConfig:
    """The parsed ``config.json``.  Sizes and constants have no defaults: what the file does not give is an error
    (``token_side``, a mixer's ``mask``, ``kv_from`` and ``rot.scaling``, and a layer's ``mlp`` may be absent or null: then
    the model has none)."""

    width: int
    vocab: int
    eps: float
    embed_scale: float
    alpha: float
    layers: List[Dict[str, Any]]
    side_dim: Optional[int] = None
    architecture: str = "Vezidra"
    eos_token_id: Optional[int] = None
    raw: Dict[str, Any] = field(default_factory=dict, repr=False)

    @classmethod
    def from_dict(cls, raw: Dict[str, Any]) -> "VezidraConfig":
        _need(raw, ("width", "vocab", "norm", "embedding", "postln_alpha", "layers"), "the top level")
        _positive(raw, ("width", "vocab"), "the top level")
        _need(raw["norm"], ("eps",), "norm")
        _need(raw["embedding"], ("scale",), "embedding")
        side = None
        if raw.get("token_side") is not None:
            _need(raw["token_side"], ("dim",), "token_side")
            _positive(raw["token_side"], ("dim",), "token_side")
            side = int(raw["token_side"]["dim"])
        layers = raw["layers"]
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: layers must be a non-empty list")
        for i, layer in enumerate(layers):
            where = f"layers[{i}]"
            _need(layer, ("type", "mixer"), where)
            kind, m = layer["type"], layer["mixer"]
            if kind not in MIXER_TYPES:
                raise ConfigError(f"config.json: {where} has type {kind!r}; known: {', '.join(MIXER_TYPES)}")
            if kind == "attention":
                _check_attention(m, f"{where}.mixer", ())
                if m.get("kv_from") is not None:
                    _check_kv_from(layers, i, where)
            else:
                _need(m, ("left", "right"), f"{where}.mixer")
                right, at = m["right"], f"{where}.mixer.right"
                if kind == "parallel":
                    _need(m, ("left_scale", "right_scale"), f"{where}.mixer")
                    _check_attention(m["left"], f"{where}.mixer.left", BY_WAVELENGTH)
                    sizes = ("heads", "kv_heads", "dim", "vdim", "conv")
                    shared = "kv_heads"
                else:
                    _check_attention(m["left"], f"{where}.mixer.left", BY_RAMP)
                    sizes = ("heads", "vdim", "state", "groups", "norm_groups", "conv")
                    shared = "groups"
                _need(right, sizes, at)
                _positive(right, sizes, at)
                if int(right["heads"]) % int(right[shared]):
                    raise ConfigError(f"config.json: {at}: heads must be a multiple of {shared}")
                if kind == "parallel_2" and int(right["heads"]) * int(right["vdim"]) % int(right["norm_groups"]):
                    raise ConfigError(f"config.json: {at}: norm_groups must divide heads * vdim")
            mlp = layer.get("mlp")
            if mlp is not None:
                _need(mlp, ("kind",), f"{where}.mlp")
                if mlp["kind"] not in MLP_KINDS:
                    raise ConfigError(f"config.json: {where}.mlp has kind {mlp['kind']!r}; known: {', '.join(MLP_KINDS)}")
                _need(mlp, ("ff",), f"{where}.mlp")
                _positive(mlp, ("ff",), f"{where}.mlp")
        return cls(width=int(raw["width"]), vocab=int(raw["vocab"]), eps=float(raw["norm"]["eps"]),
                   embed_scale=float(raw["embedding"]["scale"]), alpha=float(raw["postln_alpha"]), layers=layers,
                   side_dim=side, architecture=str(raw.get("architecture") or "Vezidra"),
                   eos_token_id=raw.get("eos_token_id"), raw=dict(raw))

    def to_dict(self) -> Dict[str, Any]:
        return dict(self.raw)


def _store_name(name: str) -> str:
    """Canonical name (``l0.mix.q.weight``, ``l2.mix.left.q.bias``) -> the file's (``l0.mix.q``, ``l2.mix.left.q.b``)."""
    if name.endswith(".weight"):
        return name[:-len(".weight")]
    if name.endswith(".bias"):
        return name[:-len(".bias")] + ".b"
    return name


def _map_name(name: str) -> str:
    if name.endswith(".b") and not name.endswith(".mix.right.b"):
        return name[:-2] + ".bias"
    return name + ".weight"


def _window(m: Dict[str, Any]) -> Optional[int]:
    return int(m["mask"]["size"]) if m.get("mask") is not None else None


def retained_keys(layers: List[Dict[str, Any]]) -> Dict[int, Optional[int]]:
    """For every attention layer that owns a cache: how many keys back its pages must stay, the longest window among
    itself and the layers that read its cache (None: one of them sees all keys)."""
    keep: Dict[int, Optional[int]] = {}
    for i, layer in enumerate(layers):
        if layer["type"] != "attention":
            continue
        owner = layer["mixer"].get("kv_from")
        owner = i if owner is None else int(owner)
        window = _window(layer["mixer"])
        if owner not in keep:
            keep[owner] = window
        elif keep[owner] is not None:
            keep[owner] = None if window is None else max(keep[owner], window)
    return keep


def _attention_spec(m: Dict[str, Any], width: int, eps: float, kind: str, retain: Optional[int]) -> PartSpec:
    """``kind``: the layer's type (the left mixer of a layer with two)."""
    rot, scaling = m["rot"], m["rot"].get("scaling") or None
    if scaling and kind == "parallel":
        scaling = {k: scaling[k] for k in BY_WAVELENGTH}
    elif scaling:
        scaling = {"kind": "ramp", **{k: scaling[k] for k in BY_RAMP}}
    position = PartSpec("rope", {"theta": float(rot["base"]), "rotary_dim": int(rot["dims"]), "scaling": scaling,
                                 "interleaved": kind != "parallel"})
    return PartSpec("paged_attention", {
        "hidden_size": width, "num_heads": int(m["heads"]), "num_kv_heads": int(m["kv_heads"]), "head_dim": int(m["dim"]),
        "value_dim": int(m["vdim"]), "qkv_bias": kind == "parallel_2", "scale": float(m["scale"]), "window": _window(m),
        "retain": retain, "qk_norm_eps": eps, "qk_norm_scope": "head" if kind == "attention" else "whole",
        "sinks": kind != "parallel_2", "plus_one": kind == "parallel_2", "head_gate": kind != "parallel_2",
        "kv_shared": m.get("kv_from") is not None, "position": position,
        "names": {"q": "q", "k": "k", "v": "v", "o": "o", "g": "g", "q_norm": "q.norm", "k_norm": "k.norm", "sink": "sink"}})


def _mixer_spec(kind: str, m: Dict[str, Any], width: int, eps: float, retain: Optional[int]) -> PartSpec:
    if kind == "attention":
        return _attention_spec(m, width, eps, kind, retain)
    r = m["right"]
    left = _attention_spec(m["left"], width, eps, kind, _window(m["left"]))
    if kind == "parallel":
        right = PartSpec("gated_delta", {
            "hidden_size": width, "num_heads": int(r["heads"]), "num_kv_heads": int(r["kv_heads"]), "key_dim": int(r["dim"]),
            "value_dim": int(r["vdim"]), "conv_taps": int(r["conv"]), "eps": eps, "unit_floor": UNIT_FLOOR,
            "names": {"q_conv": "q.conv", "k_conv": "k.conv", "v_conv": "v.conv", "a_log": "A_log"}})
        return PartSpec("side_by_side", {
            "hidden_size": width, "eps": eps, "left": left, "right": right, "norm": False,
            "factors": (float(m["left_scale"]), float(m["right_scale"]))})
    right = PartSpec("state_space_dual", {
        "hidden_size": width, "num_heads": int(r["heads"]), "value_dim": int(r["vdim"]), "state_size": int(r["state"]),
        "groups": int(r["groups"]), "norm_groups": int(r["norm_groups"]), "conv_taps": int(r["conv"]), "eps": eps,
        "names": {"a_log": "A_log", "d": "D"}})
    return PartSpec("side_by_side", {
        "hidden_size": width, "eps": eps, "factor": 0.5, "left": left, "right": right,
        "names": {"left_norm": "left.out", "right_norm": "right.out"}})


def vezidra_spec(config: VezidraConfig) -> ModelSpec:
    width, eps, dim = config.width, config.eps, config.side_dim
    norm = PartSpec("layer_norm", {"size": width, "eps": eps, "bias": True})
    keep = retained_keys(config.layers)
    layers: List[LayerSpec] = []
    run: List[RunEntry] = []
    for i, layer in enumerate(config.layers):
        m, mlp = layer["mixer"], layer.get("mlp")
        owner = m.get("kv_from") if layer["type"] == "attention" else None
        retain = keep.get(i if owner is None else int(owner))
        block = PartSpec("sum_norm", {
            "alpha": config.alpha, "mixer": _mixer_spec(layer["type"], m, width, eps, retain), "norm1": norm,
            "ffn": None if mlp is None else PartSpec("plain", {
                "hidden_size": width, "intermediate_size": int(mlp["ff"]), "activation": "relu2",
                "names": {"up": "up", "down": "down"}}),
            "norm2": norm,
            "side": None if dim is None else PartSpec("token_side", {"hidden_size": width, "dim": dim, "first": i * dim}),
            "side_norm": PartSpec("rms_norm", {"size": width, "eps": eps}),
            "names": {"mixer": "mix", "norm1": "norm1", "ffn": "mlp", "norm2": "norm2", "side": "side",
                      "side_norm": "side.norm"}})
        layers.append(LayerSpec(block, f"l{i}."))
        run.append(RunEntry(i, cache_from=None if owner is None else int(owner)))   # one entry a layer: indices agree
    sizes = {"vocab_size": config.vocab, "hidden_size": width}
    # a layer without a feed-forward has no second norm: a file that stores one all the same is read
    unused = {f"l{i}.{name}" for i, layer in enumerate(config.layers) if layer.get("mlp") is None
              for name in ("norm2", "norm2.b")}
    return ModelSpec(
        hidden_size=width, vocab_size=config.vocab, layers=layers, run=run, final_norm=norm, tie_word_embeddings=False,
        position_rows=1, embed_name="embed.weight", final_norm_prefix="final.norm.", head_name="head.weight",
        map_name=lambda name: None if name in unused else _map_name(name), store_name=_store_name,
        eos_token_id=config.eos_token_id, embed=PartSpec("token_table", {**sizes, "scale": config.embed_scale}),
        token_side_name=None if dim is None else "side.embed.weight",
        token_side_columns=0 if dim is None else dim * len(layers),
    )


register_architecture("Vezidra", vezidra_spec, VezidraConfig.from_dict)
