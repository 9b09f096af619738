"""Small Vezidra configurations and model folders with random weights for the tests.  The weights are drawn here
(not by the engine) and written with the safetensors package."""

from __future__ import annotations

import json
import os
from typing import Dict, Optional

import torch


def heads(n, kv, dim, vdim, base=10000.0, dims=None, scale=None, scaling=None, window=None, kv_from=None):
    m = {"heads": n, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5,
         "rot": {"base": base, "dims": dim if dims is None else dims}}
    if scaling is not None:
        m["rot"]["scaling"] = scaling
    if window is not None:
        m["mask"] = {"size": window}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def waves(factor=8.0, low=1.0, high=4.0, original=64):
    return {"factor": factor, "low": low, "high": high, "original": original}


def ramp(factor=4.0, original=64, fast=8.0, slow=1.0):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


def delta(n, kv, dim, vdim, conv):
    return {"heads": n, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}


def dual(n, vdim, state, groups, norm_groups, conv):
    return {"heads": n, "vdim": vdim, "state": state, "groups": groups, "norm_groups": norm_groups, "conv": conv}


def attention(m):
    return {"type": "attention", "mixer": m}


def parallel(left, right, left_scale=0.7, right_scale=1.3):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}}


def parallel_2(left, right):
    return {"type": "parallel_2", "mixer": {"left": left, "right": right}}


def layer(mixer, ff=None):
    return {**mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(width, vocab, layers, side=6, eps=1e-5, scale=3.0, alpha=2.0):
    cfg = {"architecture": "Vezidra", "width": width, "vocab": vocab, "norm": {"eps": eps}, "embedding": {"scale": scale},
           "postln_alpha": alpha, "layers": layers}
    if side is not None:
        cfg["token_side"] = {"dim": side}
    return cfg


# Sizes that all differ from one another: key/value groups of 1 and 3 heads, values wider and narrower than keys,
# partial rotation, windows of 21 and 37 (the longer one over another layer's cache) and none (pages have 16), two, three
# and four taps, every mixer with and without a feed-forward.
MIXED = config(72, 203, [
    layer(parallel(heads(6, 2, 24, 16, 80.0, 16, 0.25, waves()), delta(4, 2, 12, 20, 3)), 88),
    layer(attention(heads(4, 2, 16, 24, 500.0, 8, 0.4, window=21))),
    layer(parallel_2(heads(4, 4, 16, 24, 300.0, 12, 0.3, ramp()), dual(6, 8, 24, 3, 4, 4)), 56),
    layer(attention(heads(4, 2, 16, 24, 500.0, 8, 0.45, window=37, kv_from=1)), 40),
    layer(parallel_2(heads(3, 1, 32, 32, 900.0, 32, 0.2, ramp(2.0, 40, 4.0, 0.5)), dual(2, 40, 16, 1, 8, 2))),
    layer(parallel(heads(2, 2, 48, 48, 60.0, 48, 0.15, waves(3.0, 0.5, 2.0, 100)), delta(3, 1, 32, 16, 2), 1.1, 0.4)),
    layer(attention(heads(5, 1, 32, 32, 40.0, 20, 0.3, window=9)), 24),
], side=6)

# The same shapes with score scales so large that the softmax picks single keys: a key lost at a window's edge or a
# page's border moves the logits.
SHARP = json.loads(json.dumps(MIXED))
for _i, _s in ((0, 2.0), (1, 3.0), (2, 2.0), (3, 3.0), (4, 1.5), (5, 1.0), (6, 2.0)):
    _m = SHARP["layers"][_i]["mixer"]
    _m.get("left", _m)["scale"] = _s

# Values that happen to be 1 or equal: one head, windows of one token, one tap (a convolution without a state), one state,
# one group, one side channel, an alpha, scales and an embedding scale of 1, a wave factor of 1.
ONES = config(32, 61, [
    layer(parallel(heads(1, 1, 8, 8, 100.0, scale=1.0, scaling=waves(1.0)), delta(1, 1, 1, 1, 1), 1.0, 1.0), 32),
    layer(attention(heads(1, 1, 8, 8, 9.0, 2, 1.0, window=1)), 1),
    layer(parallel_2(heads(2, 2, 16, 16, 9.0, 16, scaling=ramp(1.0)), dual(1, 1, 1, 1, 1, 1))),
    layer(attention(heads(1, 1, 8, 8, 9.0, 2, 1.0, window=1, kv_from=1))),
    layer(parallel_2(heads(1, 1, 32, 32, 50.0), dual(4, 8, 8, 4, 1, 2)), 32),
], side=1, eps=1e-6, scale=1.0, alpha=1.0)

# Sizes that no vector width divides: odd heads, key, value, state and feed-forward sizes, five taps, nothing rotated in one
# layer's keys, no side input.
ODD = config(50, 101, [
    layer(parallel_2(heads(3, 1, 10, 14, 77.0, 6, 0.5, ramp(4.0, 30, 3.0, 0.7)), dual(3, 9, 37, 1, 3, 5)), 27),
    layer(attention(heads(2, 1, 7, 6, 50.0, 0, 0.6, window=5)), 11),
    layer(parallel(heads(3, 3, 9, 5, 50.0, 4, 0.6), delta(3, 3, 37, 7, 5), 0.3, 2.0), 9),
    layer(attention(heads(2, 1, 7, 6, 50.0, 0, 0.7, kv_from=1))),           # all keys, over a windowed layer's cache
], side=None, alpha=0.7, scale=5.0)

# Attention heads as wide as a model's: the matrix-core kernels for prompts, with sinks and without; key sizes of 64, 128
# and 80 in the recurrences.
WIDE = config(128, 157, [
    layer(attention(heads(4, 2, 128, 128, 1000.0, 64, 0.1, window=50)), 96),
    layer(parallel(heads(3, 1, 64, 64, 500.0, 64, 0.12, waves()), delta(2, 1, 128, 48, 4)), 64),
    layer(parallel_2(heads(2, 2, 96, 96, 500.0, 96, 0.1, ramp()), dual(4, 32, 80, 2, 2, 3)), 64),
    layer(parallel(heads(2, 2, 16, 16, 500.0), delta(2, 2, 64, 64, 4)), 64),
], side=32)


def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    w = cfg["width"]
    shapes = {"embed": (cfg["vocab"], w), "final.norm": (w,), "final.norm.b": (w,), "head": (cfg["vocab"], w)}
    side = (cfg.get("token_side") or {}).get("dim")
    if side:
        shapes["side.embed"] = (cfg["vocab"], side * len(cfg["layers"]))

    def attn(q, m, whole, bias, gate):
        h, g, d, v = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        shapes.update({q + "q": (h * d, w), q + "o": (w, h * v), q + "q.norm": (h * d if whole else d,)})
        if m.get("kv_from") is None:
            shapes.update({q + "k": (g * d, w), q + "v": (g * v, w), q + "k.norm": (g * d if whole else d,)})
        if bias:
            shapes.update({q + "q.b": (h * d,), q + "k.b": (g * d,), q + "v.b": (g * v,)})
        if gate:
            shapes.update({q + "g": (h, w), q + "sink": (h,)})

    for i, lay in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lay["mixer"]
        shapes.update({p + "norm1": (w,), p + "norm1.b": (w,)})
        if lay["type"] == "attention":
            attn(p + "mix.", m, False, False, True)
        elif lay["type"] == "parallel":
            attn(p + "mix.left.", m["left"], True, False, True)
            r, q = m["right"], p + "mix.right."
            gd, hv = r["kv_heads"] * r["dim"], r["heads"] * r["vdim"]
            for s, rows in (("q", gd), ("k", gd), ("v", hv)):
                shapes.update({q + s: (rows, w), f"{q}{s}.conv": (rows, r["conv"])})
            shapes.update({q + "b": (r["heads"], w), q + "a": (r["heads"], w), q + "A_log": (r["heads"],),
                           q + "dt_bias": (r["heads"],), q + "norm": (r["vdim"],), q + "g": (hv, w), q + "o": (w, hv)})
        else:
            attn(p + "mix.left.", m["left"], True, True, False)
            r, q = m["right"], p + "mix.right."
            inner, gn = r["heads"] * r["vdim"], r["groups"] * r["state"]
            shapes.update({q + "in": (2 * inner + 2 * gn + r["heads"], w), q + "conv": (inner + 2 * gn, r["conv"]),
                           q + "conv.b": (inner + 2 * gn,), q + "dt_bias": (r["heads"],), q + "A_log": (r["heads"],),
                           q + "D": (r["heads"],), q + "norm": (inner,), q + "o": (w, inner),
                           p + "mix.left.out": (w,), p + "mix.right.out": (w,)})
        if lay.get("mlp"):
            ff = lay["mlp"]["ff"]
            shapes.update({p + "norm2": (w,), p + "norm2.b": (w,), p + "mlp.up": (ff, w), p + "mlp.down": (w, ff)})
        if side:
            shapes.update({p + "side.gate": (side, w), p + "side.proj": (w, side), p + "side.norm": (w,)})
    return shapes


def random_tensors(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """bfloat16 tensors.  Matrices N(0, 1/in); gains around one; biases and sinks of both signs; decays from nearly one to
    small; step inputs and betas spread widely."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.rsplit(".", 1)[-1]
        r = torch.randn(shape, generator=g)
        if last == "b" and len(shape) == 1:
            t = 0.3 * r
        elif last in ("norm", "norm1", "norm2", "out", "D"):
            t = 1.0 + 0.25 * r
        elif last == "conv":
            t = 0.6 * r
        elif last == "sink":
            t = r
        elif last == "dt_bias":
            t = -1.0 + r
        elif last == "A_log":
            t = -0.5 + 1.2 * r
        elif name in ("embed", "side.embed"):
            t = r
        else:
            t = r / shape[1] ** 0.5
        out[name] = t.to(torch.bfloat16)
    return out


def write_model(folder: str, cfg: dict, seed: int, tensors: Optional[Dict[str, torch.Tensor]] = None) -> str:
    from safetensors.torch import save_file

    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as fh:
        json.dump(cfg, fh)
    save_file(tensors if tensors is not None else random_tensors(cfg, seed), os.path.join(folder, "model.safetensors"))
    return folder
