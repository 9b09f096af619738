"""A plain, slow implementation of the Vezidra decoder: whole sequences, token loops, no cache, dense masks, one
function per mechanism, on the CPU.  It reads config.json and the safetensors file by itself and shares no code
with the engine; the engine's logits are compared with it.

Notation: ``x`` is ``[T, width]``, a linear weight is ``[out, in]`` and applied as ``x @ W.T``.  ``store`` is
applied to whatever the engine may keep in bfloat16 (what a matrix product reads and gives, the short
convolutions' results); norms, angles, scores, softmax weights, decays, step sizes, gates of a recurrence, unit
norms, recurrent states and the residual sum stay in the working precision.
"""

from __future__ import annotations

import json
import math
import os
from typing import Callable, Dict, List, Optional

import torch

UNIT_FLOOR = 1e-6       # under the root of a unit vector's sum of squares


def _keep(x: torch.Tensor) -> torch.Tensor:
    return x


def to_bfloat16_and_back(x: torch.Tensor) -> torch.Tensor:
    return x.to(torch.bfloat16).to(x.dtype)


def vezidra_read(model_dir: str, dtype=torch.float64):
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


def layer_norm(x: torch.Tensor, w: torch.Tensor, b: torch.Tensor, eps: float) -> torch.Tensor:
    d = x - x.mean(dim=-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(dim=-1, keepdim=True) + eps) * w + b


def unit_vector(x: torch.Tensor) -> torch.Tensor:
    """The last axis divided by its length."""
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + UNIT_FLOOR)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def causal_conv(u: torch.Tensor, w: torch.Tensor, b: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``y_t = [b +] sum_j w[:, j] u_(t - taps + 1 + j)`` per channel, zeros before the first row; ``w [C, taps]``."""
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u], dim=0)
    y = torch.zeros_like(u) if b is None else torch.zeros_like(u) + b
    for j in range(taps):
        y = y + padded[j:j + u.shape[0]] * w[:, j]
    return y


# --------------------------------------------------------------------------------------------
# rotation
# --------------------------------------------------------------------------------------------
def frequencies(base: float, dims: int) -> torch.Tensor:
    """``base^(-2i/dims)``, ``i < dims/2``, in float64."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    return float(base) ** (-2.0 * i / max(dims, 1))


def by_wavelength(freqs: torch.Tensor, s: dict) -> torch.Tensor:
    """Long wavelengths stretched by ``factor``, short ones kept, a blend between."""
    out = []
    for f in freqs.tolist():
        wave = 2.0 * math.pi / f
        if wave < s["original"] / s["high"]:
            out.append(f)
        elif wave > s["original"] / s["low"]:
            out.append(f / s["factor"])
        else:
            u = (s["original"] / wave - s["low"]) / (s["high"] - s["low"])
            out.append((1.0 - u) * f / s["factor"] + u * f)
    return torch.tensor(out, dtype=torch.float64)


def by_ramp(freqs: torch.Tensor, base: float, dims: int, s: dict):
    """A ramp over the index from kept to divided frequencies; and the factor on cosines and sines."""
    def index(turns):
        return dims * math.log(s["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(index(s["fast"])), 0)
    hi = min(math.ceil(index(s["slow"])), dims - 1)
    out = []
    for i, f in enumerate(freqs.tolist()):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / s["factor"] * r + f * (1.0 - r))
    return torch.tensor(out, dtype=torch.float64), 0.1 * math.log(s["factor"]) + 1.0


def rotate(x: torch.Tensor, pos: torch.Tensor, freqs: torch.Tensor, neighbours: bool, amplitude: float = 1.0) -> torch.Tensor:
    """``x [T, heads, d]``: the first ``2 len(freqs)`` channels turned in pairs by ``pos * freqs``: channel 2i with
    2i + 1 (``neighbours``) or i with i + len(freqs); cosines and sines times ``amplitude``."""
    half = freqs.shape[0]
    if half == 0:
        return x
    angle = pos.to(torch.float64)[:, None] * freqs[None, :]
    c = (torch.cos(angle) * amplitude).to(x.dtype)[:, None, :]
    s = (torch.sin(angle) * amplitude).to(x.dtype)[:, None, :]
    first = slice(0, 2 * half, 2) if neighbours else slice(0, half)
    second = slice(1, 2 * half, 2) if neighbours else slice(half, 2 * half)
    u, v = x[..., first], x[..., second]
    out = x.clone()
    out[..., first] = u * c - v * s
    out[..., second] = v * c + u * s
    return out


# --------------------------------------------------------------------------------------------
# attention
# --------------------------------------------------------------------------------------------
def attend(q, k, v, scale: float, window: Optional[int], sink: Optional[torch.Tensor]) -> torch.Tensor:
    """``q [T, H, d]``, ``k [T, G, d]``, ``v [T, G, dv]`` -> ``[T, H, dv]``.  Query i sees the keys
    ``0 <= i - j < window`` (None: all j <= i); ``sink [H]`` (None: nothing): one more term in the denominator."""
    t, heads = q.shape[0], q.shape[1]
    per = heads // k.shape[1]
    back = torch.arange(t)[:, None] - torch.arange(t)[None, :]
    seen = back >= 0
    if window is not None:
        seen = seen & (back < window)
    out = torch.zeros(t, heads, v.shape[-1], dtype=q.dtype)
    for h in range(heads):
        s = ((q[:, h] @ k[:, h // per].T) * scale).masked_fill(~seen, -math.inf)
        top = s.max(dim=-1, keepdim=True).values
        if sink is not None:
            top = torch.maximum(top, sink[h].to(s.dtype))
        e = torch.exp(s - top)
        total = e.sum(dim=-1, keepdim=True)
        if sink is not None:
            total = total + torch.exp(sink[h].to(s.dtype) - top)
        out[:, h] = (e / total) @ v[:, h // per]
    return out


def project(h, t, name: str, store: Callable):
    y = h @ t[name].T
    return store(y + t[name + ".b"]) if name + ".b" in t else store(y)


def attention_qkv(h, pos, t, p: str, m: dict, eps: float, whole: bool, neighbours: bool, store: Callable):
    """Queries, keys and values of a layer; ``(k, v)`` None where it has no projections of them."""
    n, heads, groups, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    rot = m["rot"]
    f, amplitude = frequencies(rot["base"], rot["dims"]), 1.0
    if rot.get("scaling"):
        if "fast" in rot["scaling"]:
            f, amplitude = by_ramp(f, rot["base"], rot["dims"], rot["scaling"])
        else:
            f = by_wavelength(f, rot["scaling"])

    def normed(y, count, name):
        if whole:
            y = (unit_rms(y, eps) * t[name]).view(n, count, d)
        else:
            y = unit_rms(y.view(n, count, d), eps) * t[name]
        return store(rotate(y, pos, f, neighbours, amplitude))

    q = normed(project(h, t, p + "q", store), heads, p + "q.norm")
    if p + "k" not in t:
        return q, None, None
    k = normed(project(h, t, p + "k", store), groups, p + "k.norm")
    return q, k, project(h, t, p + "v", store).view(n, groups, m["vdim"])


def gated_by_head(o, h, w, store: Callable):
    """``o [T, H, dv]`` times the sigmoid of one number per head."""
    return o * torch.sigmoid(h @ w.T)[:, :, None]


def attention(h, pos, t, p: str, m: dict, eps: float, store: Callable = _keep, kept: Optional[dict] = None, i: int = 0):
    """A norm per head, neighbours turned, a window, a sink per head, a gate per head.  ``kept``: keys and values by
    layer; a layer with ``kv_from`` reads another's."""
    q, k, v = attention_qkv(h, pos, t, p, m, eps, False, True, store)
    kept = {} if kept is None else kept
    if m.get("kv_from") is None:
        kept[i] = (k, v)
    else:
        k, v = kept[m["kv_from"]]
    window = m["mask"]["size"] if m.get("mask") else None
    o = attend(q, k, v, m["scale"], window, t[p + "sink"])
    o = store(gated_by_head(store(o), h, t[p + "g"], store))
    return o.reshape(h.shape[0], -1) @ t[p + "o"].T


def left_with_sink(h, pos, t, p: str, m: dict, eps: float, store: Callable = _keep):
    q, k, v = attention_qkv(h, pos, t, p, m, eps, True, False, store)
    o = attend(q, k, v, m["scale"], None, t[p + "sink"])
    o = store(gated_by_head(store(o), h, t[p + "g"], store))
    return o.reshape(h.shape[0], -1) @ t[p + "o"].T


def left_plus_one(h, pos, t, p: str, m: dict, eps: float, store: Callable = _keep):
    q, k, v = attention_qkv(h, pos, t, p, m, eps, True, True, store)
    o = store(attend(q, k, v, m["scale"], None, torch.zeros(m["heads"], dtype=q.dtype)))
    return o.reshape(h.shape[0], -1) @ t[p + "o"].T


# --------------------------------------------------------------------------------------------
# recurrences
# --------------------------------------------------------------------------------------------
def delta_rule(q, k, v, decay, beta, state=None):
    """Per head ``S <- a S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q``, token by token.
    ``q, k [T, H, d]``, ``v [T, H, dv]``, ``decay, beta [T, H]``; ``(o [T, H, dv], last S [H, d, dv])``."""
    t, heads, d = q.shape
    S = torch.zeros(heads, d, v.shape[-1], dtype=q.dtype) if state is None else state.clone()
    out = torch.zeros(t, heads, v.shape[-1], dtype=q.dtype)
    for i in range(t):
        S = decay[i][:, None, None] * S
        u = beta[i][:, None] * (v[i] - (S * k[i][:, :, None]).sum(dim=1))
        S = S + k[i][:, :, None] * u[:, None, :]
        out[i] = (S * q[i][:, :, None]).sum(dim=1)
    return out, S


def decayed_products(c, b, x, decay, step, state=None):
    """Per head ``S <- a S + step b x^T; y = S^T c``, token by token (shapes as above)."""
    t, heads, n = c.shape
    S = torch.zeros(heads, n, x.shape[-1], dtype=c.dtype) if state is None else state.clone()
    out = torch.zeros(t, heads, x.shape[-1], dtype=c.dtype)
    for i in range(t):
        S = decay[i][:, None, None] * S + (step[i][:, None] * b[i])[:, :, None] * x[i][:, None, :]
        out[i] = (S * c[i][:, :, None]).sum(dim=1)
    return out, S


def spread(x: torch.Tensor, heads: int) -> torch.Tensor:
    """``[T, G, d]`` -> ``[T, heads, d]``: head h gets group ``h // (heads / G)``."""
    return x.repeat_interleave(heads // x.shape[1], dim=1)


def gated_delta(h, t, p: str, m: dict, eps: float, store: Callable = _keep):
    n, heads, groups, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (store(silu(causal_conv(store(h @ t[p + s].T), t[p + s + ".conv"]))) for s in "qkv")
    q = unit_vector(q.view(n, groups, d)) * d ** -0.5
    k = unit_vector(k.view(n, groups, d))
    beta = torch.sigmoid(h @ t[p + "b"].T)
    decay = torch.exp(-torch.exp(t[p + "A_log"]) * softplus(h @ t[p + "a"].T + t[p + "dt_bias"]))
    o, _ = delta_rule(spread(q, heads), spread(k, heads), v.view(n, heads, dv), decay, beta)
    o = (unit_rms(o, eps) * t[p + "norm"]).reshape(n, heads * dv)
    return store(o * silu(store(h @ t[p + "g"].T))) @ t[p + "o"].T


def norm_in_parts(y: torch.Tensor, parts: int, eps: float) -> torch.Tensor:
    return unit_rms(y.reshape(*y.shape[:-1], parts, -1), eps).reshape(y.shape)


def state_space_dual(h, t, p: str, m: dict, eps: float, store: Callable = _keep):
    n, heads, dv, states, groups = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner, gn = heads * dv, groups * states
    proj = h @ t[p + "in"].T
    z = store(proj[:, :inner])
    xbc = store(silu(causal_conv(store(proj[:, inner:2 * inner + 2 * gn]), t[p + "conv"], t[p + "conv.b"])))
    x = xbc[:, :inner].view(n, heads, dv)
    b = spread(xbc[:, inner:inner + gn].view(n, groups, states), heads)
    c = spread(xbc[:, inner + gn:].view(n, groups, states), heads)
    step = softplus(proj[:, 2 * inner + 2 * gn:] + t[p + "dt_bias"])
    y, _ = decayed_products(c, b, x, torch.exp(-torch.exp(t[p + "A_log"]) * step), step)
    y = (y + t[p + "D"][None, :, None] * x).reshape(n, inner) * silu(z)
    return store(norm_in_parts(y, m["norm_groups"], eps) * t[p + "norm"]) @ t[p + "o"].T


# --------------------------------------------------------------------------------------------
# layers
# --------------------------------------------------------------------------------------------
def parallel(h, pos, t, p: str, m: dict, eps: float, store: Callable = _keep):
    left = store(left_with_sink(h, pos, t, p + "left.", m["left"], eps, store))
    right = store(gated_delta(h, t, p + "right.", m["right"], eps, store))
    return m["left_scale"] * left + m["right_scale"] * right


def parallel_2(h, pos, t, p: str, m: dict, eps: float, store: Callable = _keep):
    left = store(left_plus_one(h, pos, t, p + "left.", m["left"], eps, store))
    right = store(state_space_dual(h, t, p + "right.", m["right"], eps, store))
    return 0.5 * (unit_rms(left, eps) * t[p + "left.out"] + unit_rms(right, eps) * t[p + "right.out"])


def mixer(kind: str, h, pos, t, p: str, m: dict, eps: float, store: Callable, kept: dict, i: int):
    if kind == "attention":
        return store(attention(h, pos, t, p, m, eps, store, kept, i))
    return {"parallel": parallel, "parallel_2": parallel_2}[kind](h, pos, t, p, m, eps, store)


def squared_relu_ff(x, t, p: str, store: Callable = _keep):
    z = store(x @ t[p + "up"].T)
    return store(torch.clamp(z, min=0.0) ** 2) @ t[p + "down"].T


def side_input(x, rows, t, p: str, eps: float, store: Callable = _keep):
    """What a layer's own rows of the second table (``rows [T, dim]``) add, gated by ``x``."""
    g = store(gelu_tanh(x @ t[p + "gate"].T) * rows)
    return unit_rms(store(g @ t[p + "proj"].T), eps) * t[p + "norm"]


def layer(cfg: dict, t, i: int, x, tokens, pos, kept: dict, store: Callable = _keep):
    lay, eps, alpha, p = cfg["layers"][i], cfg["norm"]["eps"], cfg["postln_alpha"], f"l{i}."
    y = mixer(lay["type"], store(x), pos, t, p + "mix.", lay["mixer"], eps, store, kept, i)
    x = layer_norm(alpha * x + y, t[p + "norm1"], t[p + "norm1.b"], eps)
    if lay.get("mlp") is not None:
        y = store(squared_relu_ff(store(x), t, p + "mlp.", store))
        x = layer_norm(alpha * x + y, t[p + "norm2"], t[p + "norm2.b"], eps)
    if cfg.get("token_side"):
        dim = cfg["token_side"]["dim"]
        rows = t["side.embed"][torch.tensor(tokens)][:, i * dim:(i + 1) * dim]
        x = x + side_input(store(x), rows, t, p + "side.", eps, store)
    return x


def embed(cfg: dict, t, tokens: List[int]) -> torch.Tensor:
    return t["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]


def vezidra_forward(cfg: dict, t: Dict[str, torch.Tensor], tokens: List[int], store: Callable = _keep,
                    trace: Optional[list] = None):
    """Logits ``[T, vocab]`` of a whole sequence; ``trace`` collects the residual sum after every layer."""
    pos = torch.arange(len(tokens))
    x, kept = embed(cfg, t, tokens), {}
    for i in range(len(cfg["layers"])):
        x = layer(cfg, t, i, x, tokens, pos, kept, store)
        if trace is not None:
            trace.append(x)
    x = layer_norm(x, t["final.norm"], t["final.norm.b"], cfg["norm"]["eps"])
    return store(x) @ t["head"].T
