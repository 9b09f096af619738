"""The Zaposun decoder as a model spec.

The stream starts at ``table[id] + pairs[(previous id * mul_prev + id * mul_cur) mod buckets]`` (the last row of
``pairs`` for a sequence's first token) in every one of ``streams`` copies of the residual sum.  A layer is pre-normed;
each of its sublayers reads a weighted sum of the copies and its result joins them by a mix (hyper-connections,
:mod:`~qwen25vl_lite_amd.parts.hyper`).  The norms divide each of ``norm.groups`` equal parts of a row by its own root
mean square.  What a mixer reads is first moved towards the previous token's by a weight per channel.  Two mixers:

* ``wkv``: a recurrence over outer products with a decay per token and key channel and a bonus for the current
  token, whose five projections each read a mix of their own with the previous token.
* ``parallel``: half the sum of two mixers' outputs, each normed over the width.  Left, grouped attention in chunks of
  ``mask.size`` positions with an RMS norm per head on queries and keys, rotation of the first ``rot.dims`` channels in
  halves, a fixed score scale, and values that are turned by their positions and turned back behind the sum.  Right, a
  selective state space with a short convolution.

Feed-forwards: ``dense``, ``down(gelu(gate x) * up x)`` with gelu's tanh form, or none.  The final norm reads the sum of
the copies; the logits are an untied head's times ``logit_scale``.

``config.json``: ``architecture``, ``width``, ``vocab``, ``norm.eps``, ``norm.groups``, ``streams``,
``embedding.bigram`` (``buckets``, ``mul_prev``, ``mul_cur``), ``logit_scale`` and ``layers``, a list of ``{"type", "mixer":
{...}, "mlp": {...} | null}``.  Tensors are named ``embed``, ``bigram``, ``final.norm``, ``head``, ``l<i>.norm1|norm2``,
``l<i>.shift``, ``l<i>.hc1|hc2.in|out|mix``, ``l<i>.mix.<name>``, ``l<i>.mix.left|right.<name>``, ``l<i>.mlp.<name>``; a
bias ends in ``.b``.
"""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from ..config.model_config import ConfigError
from ..config.registry import register_architecture
from ..parts.base import PartSpec
from .spec import LayerSpec, ModelSpec, RunEntry

__all__ = ["ZaposunConfig", "zaposun_spec"]

MIXER_TYPES = ("parallel", "wkv")
MLP_KINDS = ("dense",)


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


def _check_left(m: Any, where: str) -> None:
    sizes = ("heads", "kv_heads", "dim", "vdim")
    _need(m, sizes + ("mask", "rot", "scale"), where)
    _positive(m, sizes, where)
    _positive(m, ("scale",), where, whole=False)
    if int(m["heads"]) % int(m["kv_heads"]):
        raise ConfigError(f"config.json: {where}: heads must be a multiple of kv_heads")
    if int(m["vdim"]) % 2:
        raise ConfigError(f"config.json: {where}: values are turned in pairs, so vdim must be even")
    _need(m["mask"], ("size",), f"{where}.mask")
    _positive(m["mask"], ("size",), f"{where}.mask")
    _need(m["rot"], ("base", "dims"), f"{where}.rot")
    _positive(m["rot"], ("base",), f"{where}.rot", whole=False)
    dims = int(m["rot"]["dims"])
    if dims < 0 or dims % 2 or dims > int(m["dim"]):
        raise ConfigError(f"config.json: {where}.rot.dims must be even and at most dim")


def _check_right(m: Any, where: str) -> None:
    sizes = ("inner", "state", "dt_rank", "conv")
    _need(m, sizes, where)
    _positive(m, sizes, where)


@dataclass
class ZaposunConfig:
    """The parsed ``config.json``.  Sizes and constants have no defaults: what the file does not give is an error
    (a layer's ``mlp`` may be absent or null: then the layer has no feed-forward)."""

    width: int
    vocab: int
    eps: float
    groups: int
    streams: int
    logit_scale: float
    bigram: Dict[str, int]
    layers: List[Dict[str, Any]]
    architecture: str = "Zaposun"
    eos_token_id: Optional[int] = None
    raw: Dict[str, Any] = field(default_factory=dict, repr=False)

    @classmethod
    def from_dict(cls, raw: Dict[str, Any]) -> "ZaposunConfig":
        _need(raw, ("width", "vocab", "norm", "embedding", "streams", "logit_scale", "layers"), "the top level")
        _positive(raw, ("width", "vocab", "streams"), "the top level")
        _need(raw["norm"], ("eps", "groups"), "norm")
        _positive(raw["norm"], ("groups",), "norm")
        if int(raw["width"]) % int(raw["norm"]["groups"]):
            raise ConfigError("config.json: norm.groups must divide width into equal parts")
        _need(raw["embedding"], ("bigram",), "embedding")
        _need(raw["embedding"]["bigram"], ("buckets", "mul_prev", "mul_cur"), "embedding.bigram")
        _positive(raw["embedding"]["bigram"], ("buckets",), "embedding.bigram")
        layers = raw["layers"]
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: layers must be a non-empty list")
        for i, layer in enumerate(layers):
            where = f"layers[{i}]"
            _need(layer, ("type", "mixer"), where)
            kind, m = layer["type"], layer["mixer"]
            if kind not in MIXER_TYPES:
                raise ConfigError(f"config.json: {where} has type {kind!r}; known: {', '.join(MIXER_TYPES)}")
            if kind == "wkv":
                _need(m, ("heads", "dim"), f"{where}.mixer")
                _positive(m, ("heads", "dim"), f"{where}.mixer")
            else:
                _need(m, ("left", "right"), f"{where}.mixer")
                _check_left(m["left"], f"{where}.mixer.left")
                _check_right(m["right"], f"{where}.mixer.right")
            mlp = layer.get("mlp")
            if mlp is not None:
                _need(mlp, ("kind",), f"{where}.mlp")
                if mlp["kind"] not in MLP_KINDS:
                    raise ConfigError(f"config.json: {where}.mlp has kind {mlp['kind']!r}; known: {', '.join(MLP_KINDS)}")
                _need(mlp, ("ff",), f"{where}.mlp")
                _positive(mlp, ("ff",), f"{where}.mlp")
        bigram = {k: int(raw["embedding"]["bigram"][k]) for k in ("buckets", "mul_prev", "mul_cur")}
        return cls(width=int(raw["width"]), vocab=int(raw["vocab"]), eps=float(raw["norm"]["eps"]),
                   groups=int(raw["norm"]["groups"]), streams=int(raw["streams"]), logit_scale=float(raw["logit_scale"]),
                   bigram=bigram, layers=layers, architecture=str(raw.get("architecture") or "Zaposun"),
                   eos_token_id=raw.get("eos_token_id"), raw=dict(raw))

    def to_dict(self) -> Dict[str, Any]:
        return dict(self.raw)


def _store_name(name: str) -> str:
    """Canonical name (``l0.mix.r.weight``, ``l1.mix.right.dt.bias``) -> the file's (``l0.mix.r``, ``l1.mix.right.dt.b``).
    The embedding's second table has a name of its own in a file."""
    if name == "embed.bigram.weight":
        return "bigram"
    if name.endswith(".weight"):
        return name[:-len(".weight")]
    if name.endswith(".bias"):
        return name[:-len(".bias")] + ".b"
    return name


def _map_name(name: str) -> str:
    if name == "bigram":
        return "embed.bigram.weight"
    return name[:-2] + ".bias" if name.endswith(".b") else name + ".weight"


def _left_spec(m: Dict[str, Any], width: int, eps: float) -> PartSpec:
    base = float(m["rot"]["base"])
    return PartSpec("paged_attention", {
        "hidden_size": width, "num_heads": int(m["heads"]), "num_kv_heads": int(m["kv_heads"]), "head_dim": int(m["dim"]),
        "value_dim": int(m["vdim"]), "qkv_bias": False, "scale": float(m["scale"]), "qk_norm_eps": eps,
        "chunk": int(m["mask"]["size"]), "value_rotation": base,
        "position": PartSpec("rope", {"theta": base, "rotary_dim": int(m["rot"]["dims"])}),
        "names": {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm"}})


def _right_spec(m: Dict[str, Any], width: int) -> PartSpec:
    return PartSpec("selective_state_space", {
        "hidden_size": width, "inner_size": int(m["inner"]), "state_size": int(m["state"]), "dt_rank": int(m["dt_rank"]),
        "conv_taps": int(m["conv"]), "names": {"a_log": "A_log", "d": "D"}})


def _mixer_spec(kind: str, m: Dict[str, Any], width: int, eps: float) -> PartSpec:
    if kind == "wkv":
        return PartSpec("time_mix", {"hidden_size": width, "num_heads": int(m["heads"]), "head_dim": int(m["dim"]), "eps": eps})
    return PartSpec("side_by_side", {
        "hidden_size": width, "eps": eps, "factor": 0.5, "left": _left_spec(m["left"], width, eps),
        "right": _right_spec(m["right"], width), "names": {"left_norm": "left.out", "right_norm": "right.out"}})


def zaposun_spec(config: ZaposunConfig) -> ModelSpec:
    width, eps = config.width, config.eps
    norm = PartSpec("copies", {"size": width, "eps": eps, "copies": config.streams, "groups": config.groups})
    layers: List[LayerSpec] = []
    for i, layer in enumerate(config.layers):
        mlp = layer.get("mlp")
        block = PartSpec("copies", {
            "copies": config.streams, "norm1": norm, "mixer": _mixer_spec(layer["type"], layer["mixer"], width, eps),
            "filter": PartSpec("token_shift", {"channels": width}),
            "norm2": None if mlp is None else norm,
            "ffn": None if mlp is None else PartSpec("swiglu", {
                "hidden_size": width, "intermediate_size": int(mlp["ff"]), "activation": "gelu_tanh",
                "names": {"gate": "gate", "up": "up", "down": "down"}}),
            "names": {"norm1": "norm1", "mixer": "mix", "norm2": "norm2", "ffn": "mlp", "filter": "shift",
                      "join1": "hc1", "join2": "hc2"}})
        layers.append(LayerSpec(block, f"l{i}."))
    sizes = {"vocab_size": config.vocab, "hidden_size": width}
    # a layer without a feed-forward has no second norm and connection: a file that stores them all the same is read
    unused = {f"l{i}.{name}" for i, layer in enumerate(config.layers) if layer.get("mlp") is None
              for name in ("norm2", "hc2.in", "hc2.out", "hc2.mix")}
    return ModelSpec(
        hidden_size=width, vocab_size=config.vocab, layers=layers, run=[RunEntry(i) for i in range(len(layers))],
        final_norm=norm, tie_word_embeddings=False, position_rows=1,
        embed_name="embed.weight", final_norm_prefix="final.norm.", head_name="head.weight",
        map_name=lambda name: None if name in unused else _map_name(name), store_name=_store_name,
        eos_token_id=config.eos_token_id,
        embed=PartSpec("bigram_table", {**sizes, **config.bigram, "pairs_name": "bigram"}),
        head=PartSpec("linear", {**sizes, "scale": config.logit_scale}),
    )


register_architecture("Zaposun", zaposun_spec, ZaposunConfig.from_dict)
