"""Small Zaposun configurations and model folders with random weights for the tests.  The weights are drawn here
(not by the engine) and written with the safetensors package."""

from __future__ import annotations

import json
import os
from typing import Dict, Optional

import torch


def left(heads, kv_heads, dim, vdim, chunk, base=10000.0, dims=None, scale=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": chunk},
            "rot": {"base": base, "dims": dim if dims is None else dims}, "scale": scale or dim ** -0.5}


def right(inner, state, dt_rank, conv):
    return {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}


def parallel(l, r):
    return {"type": "parallel", "mixer": {"left": l, "right": r}}


def wkv(heads, dim):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim}}


def layer(mixer, ff=None):
    return {**mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(width, vocab, layers, streams=2, groups=2, eps=1e-5, logit_scale=0.7, bigram=(97, 31, 7)):
    return {"architecture": "Zaposun", "width": width, "vocab": vocab, "norm": {"eps": eps, "groups": groups},
            "streams": streams, "logit_scale": logit_scale,
            "embedding": {"bigram": {"buckets": bigram[0], "mul_prev": bigram[1], "mul_cur": bigram[2]}}, "layers": layers}


# Sizes that all differ from one another: key/value groups of 1 and 3 heads, values wider and narrower than keys,
# partial rotation, chunks of 37 and 9 positions (pages have 16), two, three and four taps, layers of either kind with
# and without a feed-forward.  RANKS: the decay projections' inner sizes, which only the tensors say.
MIXED = config(72, 203, [
    layer(wkv(3, 16), 88),
    layer(parallel(left(6, 2, 24, 16, 37, base=80.0, dims=16, scale=0.25), right(88, 8, 5, 3)), 56),
    layer(parallel(left(4, 4, 16, 24, 9, base=500.0, dims=8, scale=0.4), right(40, 3, 8, 4))),
    layer(wkv(2, 32)),
    layer(parallel(left(3, 1, 16, 24, 64, base=300.0, dims=16, scale=0.3), right(64, 16, 3, 2)), 40),
], streams=3, groups=3, bigram=(61, 29, 5))
RANKS = {0: 6, 3: 24}

# The same shapes with score scales so large that the softmax picks single keys: a key lost at a chunk's edge or a
# page's border moves the logits.
SHARP = json.loads(json.dumps(MIXED))
for _i, _s in ((1, 2.0), (2, 3.0), (4, 2.0)):
    SHARP["layers"][_i]["mixer"]["left"]["scale"] = _s

# Values that happen to be 1 or equal: one stream, one group of the norm, one head, chunks of one token, one tap (a
# convolution without a state), one state a channel, a step size from one channel, one bucket, a logit scale of 1.
ONES = config(32, 61, [
    layer(parallel(left(1, 1, 8, 8, 1, base=100.0, scale=1.0), right(1, 1, 1, 1)), 32),
    layer(wkv(1, 8), 1),
    layer(parallel(left(2, 2, 16, 16, 16, base=9.0, dims=2), right(32, 1, 32, 1))),
], streams=1, groups=1, eps=1e-6, logit_scale=1.0, bigram=(1, 1, 1))

# Sizes that no vector width divides: odd head, state, inner and feed-forward sizes, parts of the norm of ten
# channels, five streams and taps, nothing rotated in one layer's keys, states shared by several waves.
ODD = config(50, 101, [
    layer(parallel(left(3, 1, 10, 14, 5, base=77.0, dims=6, scale=0.5), right(27, 35, 3, 5)), 27),
    layer(wkv(3, 5), 11),
    layer(parallel(left(2, 1, 7, 6, 23, base=50.0, dims=0, scale=0.6), right(19, 3, 2, 2)), 9),
], streams=5, groups=5, logit_scale=1.9, bigram=(1000003, 100003, 17))

# Recurrences only: no keys and values in any page.
NO_PAGES = config(40, 77, [layer(wkv(2, 20), 24), layer(wkv(5, 8))], streams=4, groups=10, bigram=(33, 2, 3))


def tensor_shapes(cfg: dict, ranks: Optional[Dict[int, int]] = None) -> Dict[str, tuple]:
    w, s, ranks = cfg["width"], cfg["streams"], ranks or {}
    shapes = {"embed": (cfg["vocab"], w), "bigram": (cfg["embedding"]["bigram"]["buckets"] + 1, w), "final.norm": (w,),
              "head": (cfg["vocab"], w)}
    for i, lay in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lay["mixer"]
        shapes.update({p + "norm1": (w,), p + "shift": (w,), p + "hc1.in": (s,), p + "hc1.out": (s,), p + "hc1.mix": (s, s)})
        if lay["type"] == "wkv":
            hd, rank = m["heads"] * m["dim"], ranks.get(i, 7)
            shapes.update({f"{p}mix.mu.{x}": (w,) for x in "rkvgw"})
            shapes.update({f"{p}mix.{x}": (hd, w) for x in "rkvg"})
            shapes.update({p + "mix.w1": (rank, w), p + "mix.w2": (hd, rank), p + "mix.w0": (hd,),
                           p + "mix.u": (m["heads"], m["dim"]), p + "mix.norm": (hd,), p + "mix.o": (w, hd)})
        else:
            a, b = m["left"], m["right"]
            h, g, d, v, c, n = a["heads"], a["kv_heads"], a["dim"], a["vdim"], b["inner"], b["state"]
            q = p + "mix.left."
            shapes.update({q + "q": (h * d, w), q + "k": (g * d, w), q + "v": (g * v, w), q + "q.norm": (d,),
                           q + "k.norm": (d,), q + "o": (w, h * v), q + "out": (w,)})
            q = p + "mix.right."
            shapes.update({q + "in": (2 * c, w), q + "conv": (c, b["conv"]), q + "conv.b": (c,),
                           q + "x": (b["dt_rank"] + 2 * n, c), q + "dt": (c, b["dt_rank"]), q + "dt.b": (c,),
                           q + "A_log": (c, n), q + "D": (c,), q + "o": (w, c), q + "out": (w,)})
        if lay.get("mlp"):
            ff = lay["mlp"]["ff"]
            shapes.update({p + "norm2": (w,), p + "hc2.in": (s,), p + "hc2.out": (s,), p + "hc2.mix": (s, s),
                           p + "mlp.gate": (ff, w), p + "mlp.up": (ff, w), p + "mlp.down": (w, ff)})
    return shapes


def random_tensors(cfg: dict, seed: int, ranks: Optional[Dict[int, int]] = None) -> Dict[str, torch.Tensor]:
    """bfloat16 tensors.  Matrices N(0, 1/in); gains around one; token mixes uniform on [0, 1); a connection's mix
    around the identity with off-diagonal entries of both signs; decays from nearly one to small."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, ranks).items():
        last = name.rsplit(".", 1)[-1]
        r = torch.randn(shape, generator=g)
        if last in ("norm", "norm1", "norm2", "D") or name.endswith((".left.out", ".right.out")):
            t = 1.0 + 0.25 * r
        elif last == "shift" or ".mu." in name:
            t = torch.rand(shape, generator=g)
        elif ".hc" in name:
            t = {"in": 0.5 + 0.4 * r, "out": 0.8 + 0.4 * r,
                 "mix": torch.eye(shape[0]) + 0.2 * r if len(shape) == 2 else r}[last]
        elif last == "w0":
            t = -1.5 + 1.5 * r
        elif last == "u" or last == "conv":
            t = 0.5 * r
        elif name.endswith("conv.b"):
            t = 0.3 * r
        elif name.endswith("dt.b"):
            t = -1.0 + r
        elif last == "A_log":
            t = torch.log(torch.arange(1, shape[1] + 1).float())[None, :] + 0.3 * r
        elif last in ("embed", "bigram"):
            t = r
        else:
            t = r / shape[1] ** 0.5
        out[name] = t.to(torch.bfloat16)
    return out


def write_model(folder: str, cfg: dict, seed: int, tensors: Optional[Dict[str, torch.Tensor]] = None,
                ranks: Optional[Dict[int, int]] = None) -> str:
    from safetensors.torch import save_file

    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as fh:
        json.dump(cfg, fh)
    save_file(tensors if tensors is not None else random_tensors(cfg, seed, ranks), os.path.join(folder, "model.safetensors"))
    return folder
