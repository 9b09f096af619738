"""A plain, slow implementation of the Zaposun decoder: whole sequences, token loops, no cache, dense masks, one
function per mechanism, on the CPU.  It reads config.json and the safetensors file by itself and shares no code
with the engine; the engine's logits are compared with it.

Notation: ``x`` is ``[T, width]``, a linear weight is ``[out, in]`` and applied as ``x @ W.T``.  ``store`` is
applied to whatever the engine may keep in bfloat16 (what a matrix product reads and gives, the short
convolution's result); norms, the mixes of neighbouring tokens, angles, scores, softmax weights, decays, step
sizes, recurrent states and the residual sums stay in the working precision.
"""

from __future__ import annotations

import json
import math
import os
from typing import Callable, Dict, List, Optional

import torch


def _keep(x: torch.Tensor) -> torch.Tensor:
    return x


def to_bfloat16_and_back(x: torch.Tensor) -> torch.Tensor:
    return x.to(torch.bfloat16).to(x.dtype)


def zaposun_read(model_dir: str, dtype=torch.float64):
    """``(config dict, {tensor name: tensor})`` with the names the file uses."""
    from safetensors import safe_open

    with open(os.path.join(model_dir, "config.json")) as fh:
        cfg = json.load(fh)
    tensors = {}
    with safe_open(os.path.join(model_dir, "model.safetensors"), framework="pt", device="cpu") as f:
        for name in f.keys():
            tensors[name] = f.get_tensor(name).to(dtype)
    return cfg, tensors


# --------------------------------------------------------------------------------------------
# small pieces
# --------------------------------------------------------------------------------------------
def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """The last axis divided by its root mean square, eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def grouped_norm(x: torch.Tensor, w: torch.Tensor, groups: int, eps: float) -> torch.Tensor:
    """Every one of ``groups`` consecutive parts of a row divided by its own root mean square, then the gains."""
    parts = x.reshape(*x.shape[:-1], groups, x.shape[-1] // groups)
    return unit_rms(parts, eps).reshape(x.shape) * w


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def one_back(h: torch.Tensor) -> torch.Tensor:
    """The rows of the tokens before; zeros before the first."""
    return torch.cat([torch.zeros_like(h[:1]), h[:-1]], dim=0)


def towards_previous(h: torch.Tensor, mu: torch.Tensor) -> torch.Tensor:
    """``h_t + (h_(t-1) - h_t) mu``, element by element."""
    return h + (one_back(h) - h) * mu


def frequencies(base: float, dims: int) -> torch.Tensor:
    """``base^(-2i/dims)``, ``i < dims/2``, in float64."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    return float(base) ** (-2.0 * i / dims)


def rotate(x: torch.Tensor, pos: torch.Tensor, freqs: torch.Tensor) -> torch.Tensor:
    """``x [T, heads, d]``: channel i of the first ``2 len(freqs)`` turned with channel i + len(freqs) by
    ``pos * freqs``; a negative ``pos`` turns back."""
    half = freqs.shape[0]
    if half == 0:
        return x
    angle = pos.to(torch.float64)[:, None] * freqs[None, :]
    c, s = torch.cos(angle).to(x.dtype)[:, None, :], torch.sin(angle).to(x.dtype)[:, None, :]
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], dim=-1)


def causal_conv(u: torch.Tensor, w: torch.Tensor, b: torch.Tensor) -> torch.Tensor:
    """``y_t = b + sum_j w[:, j] u_(t - taps + 1 + j)`` per channel, zeros before the first row; ``w [C, taps]``."""
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u], dim=0)
    y = torch.zeros_like(u) + b
    for j in range(taps):
        y = y + padded[j:j + u.shape[0]] * w[:, j]
    return y


def attend_in_chunks(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, chunk: Optional[int]) -> torch.Tensor:
    """``q [T, H, d]``, ``k [T, G, d]``, ``v [T, G, dv]`` -> ``[T, H, dv]``.  Query i sees the keys j <= i of its
    own chunk of ``chunk`` positions."""
    t, heads = q.shape[0], q.shape[1]
    per = heads // k.shape[1]
    i = torch.arange(t)
    seen = i[None, :] <= i[:, None]
    if chunk is not None:
        seen = seen & (i[None, :] // chunk == i[:, None] // chunk)
    out = torch.zeros(t, heads, v.shape[-1], dtype=q.dtype)
    for h in range(heads):
        s = (q[:, h] @ k[:, h // per].T) * scale
        e = torch.exp(s.masked_fill(~seen, -math.inf) - s.masked_fill(~seen, -math.inf).max(dim=-1, keepdim=True).values)
        out[:, h] = (e / e.sum(dim=-1, keepdim=True)) @ v[:, h // per]
    return out


# --------------------------------------------------------------------------------------------
# mixers
# --------------------------------------------------------------------------------------------
def chunked_attention(h, pos, t: Dict[str, torch.Tensor], p: str, m: dict, eps: float, store: Callable = _keep):
    """Normed and rotated queries and keys; values turned by their own position and turned back behind the sum."""
    n, heads, groups, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = store(h @ t[p + "q"].T).view(n, heads, d)
    k = store(h @ t[p + "k"].T).view(n, groups, d)
    v = store(h @ t[p + "v"].T).view(n, groups, dv)
    f = frequencies(m["rot"]["base"], m["rot"]["dims"])
    q = store(rotate(unit_rms(q, eps) * t[p + "q.norm"], pos, f))
    k = store(rotate(unit_rms(k, eps) * t[p + "k.norm"], pos, f))
    fv = frequencies(m["rot"]["base"], dv)
    v = store(rotate(v, pos, fv))
    o = rotate(attend_in_chunks(q, k, v, m["scale"], m["mask"]["size"]), -pos, fv)
    return store(o).reshape(n, heads * dv) @ t[p + "o"].T


def selective_scan(x: torch.Tensor, dt: torch.Tensor, a: torch.Tensor, b: torch.Tensor, c: torch.Tensor, d: torch.Tensor):
    """``S <- exp(dt A) S + dt x B``, ``y = S C + D x`` per channel, token by token; ``x, dt [T, C]``, ``a [C, n]``,
    ``b, c [T, n]``, ``d [C]``."""
    state = torch.zeros_like(a)
    out = torch.zeros_like(x)
    for i in range(x.shape[0]):
        state = torch.exp(dt[i][:, None] * a) * state + (dt[i] * x[i])[:, None] * b[i][None, :]
        out[i] = state @ c[i] + d * x[i]
    return out


def mamba(h, t, p: str, m: dict, store: Callable = _keep):
    inner, rank, n = m["inner"], m["dt_rank"], m["state"]
    both = store(h @ t[p + "in"].T)
    x, z = both[:, :inner], both[:, inner:]
    x = store(silu(causal_conv(x, t[p + "conv"], t[p + "conv.b"])))
    low = x @ t[p + "x"].T
    dt = softplus(store(low[:, :rank]) @ t[p + "dt"].T + t[p + "dt.b"])
    y = selective_scan(x, dt, -torch.exp(t[p + "A_log"]), low[:, rank:rank + n], low[:, rank + n:], t[p + "D"])
    return store(y * silu(z)) @ t[p + "o"].T


def parallel(h, pos, t, p: str, m: dict, eps: float, store: Callable = _keep):
    """Half the sum of the two mixers' outputs, each normed over the width."""
    left = store(chunked_attention(h, pos, t, p + "left.", m["left"], eps, store))
    right = store(mamba(h, t, p + "right.", m["right"], store))
    return 0.5 * (unit_rms(left, eps) * t[p + "left.out"] + unit_rms(right, eps) * t[p + "right.out"])


def decayed_outer_products(r, k, v, w, u):
    """``o_t = (S + diag(u) k_t v_t^T)^T r_t``, then ``S <- diag(w_t) S + k_t v_t^T``; ``[T, H, d]`` each, ``u [H, d]``."""
    t, heads, d = r.shape
    state = torch.zeros(heads, d, v.shape[-1], dtype=r.dtype)
    out = torch.zeros(t, heads, v.shape[-1], dtype=r.dtype)
    for i in range(t):
        kv = k[i][:, :, None] * v[i][:, None, :]
        out[i] = ((state + u[:, :, None] * kv) * r[i][:, :, None]).sum(dim=1)
        state = w[i][:, :, None] * state + kv
    return out


def wkv(h, pos, t, p: str, m: dict, eps: float, store: Callable = _keep):
    n, heads, d = h.shape[0], m["heads"], m["dim"]
    mixed = {s: store(towards_previous(h, t[f"{p}mu.{s}"])) for s in "rkvgw"}
    r, k, v = (store(mixed[s] @ t[p + s].T).view(n, heads, d) for s in "rkv")
    z = store(torch.tanh(mixed["w"] @ t[p + "w1"].T)) @ t[p + "w2"].T + t[p + "w0"]
    o = decayed_outer_products(r, k, v, torch.exp(-torch.exp(z)).view(n, heads, d), t[p + "u"])
    o = unit_rms(o, eps).reshape(n, heads * d) * t[p + "norm"]
    return store(o * silu(store(mixed["g"] @ t[p + "g"].T))) @ t[p + "o"].T


MIXERS = {"parallel": parallel, "wkv": wkv}


# --------------------------------------------------------------------------------------------
# the model
# --------------------------------------------------------------------------------------------
def gated_ff(x, t, p: str, store: Callable = _keep):
    return store(gelu_tanh(store(x @ t[p + "gate"].T)) * store(x @ t[p + "up"].T)) @ t[p + "down"].T


def bigram_rows(tokens: List[int], bigram: dict) -> torch.Tensor:
    """The bigram table's row for every token: the last row for a sequence's first."""
    rows, prev = [], None
    for tok in tokens:
        rows.append(bigram["buckets"] if prev is None else
                    (prev * bigram["mul_prev"] + tok * bigram["mul_cur"]) % bigram["buckets"])
        prev = tok
    return torch.tensor(rows)


def join(streams: torch.Tensor, y: torch.Tensor, t, p: str) -> torch.Tensor:
    """``streams [S, T, width]``: every stream becomes a mix of the old ones (``mix[from, to]``) plus its share of ``y``."""
    mix, out = t[p + "mix"], t[p + "out"]
    return torch.stack([sum(mix[a, b] * streams[a] for a in range(len(streams))) + out[b] * y
                        for b in range(len(streams))])


def read(streams: torch.Tensor, t, p: str) -> torch.Tensor:
    return sum(w * s for w, s in zip(t[p + "in"], streams))


def layer(cfg: dict, t, i: int, streams, pos, store: Callable = _keep):
    lay, norm, p = cfg["layers"][i], cfg["norm"], f"l{i}."
    h = grouped_norm(read(streams, t, p + "hc1."), t[p + "norm1"], norm["groups"], norm["eps"])
    h = towards_previous(h, t[p + "shift"])
    # the engine hands a recurrence's own mix of tokens the unrounded rows, other mixers the rounded ones
    h = h if lay["type"] == "wkv" else store(h)
    y = MIXERS[lay["type"]](h, pos, t, p + "mix.", lay["mixer"], norm["eps"], store)
    streams = join(streams, y, t, p + "hc1.")
    if lay.get("mlp") is not None:
        h = store(grouped_norm(read(streams, t, p + "hc2."), t[p + "norm2"], norm["groups"], norm["eps"]))
        streams = join(streams, gated_ff(h, t, p + "mlp.", store), t, p + "hc2.")
    return streams


def embed(cfg: dict, t, tokens: List[int]) -> torch.Tensor:
    return t["embed"][torch.tensor(tokens)] + t["bigram"][bigram_rows(tokens, cfg["embedding"]["bigram"])]


def zaposun_forward(cfg: dict, t, tokens: List[int], store: Callable = _keep, trace: Optional[list] = None):
    """Logits ``[T, vocab]`` of a whole sequence; ``trace`` collects the sum of the streams after every layer."""
    pos = torch.arange(len(tokens))
    streams = torch.stack([embed(cfg, t, tokens)] * cfg["streams"])
    for i in range(len(cfg["layers"])):
        streams = layer(cfg, t, i, streams, pos, store)
        if trace is not None:
            trace.append(streams.sum(0))
    x = grouped_norm(streams.sum(0), t["final.norm"], cfg["norm"]["groups"], cfg["norm"]["eps"])
    return store(x) @ t["head"].T * cfg["logit_scale"]
