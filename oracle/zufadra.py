"""CPU restatement of the Zufadra decoder (test infrastructure only): one function per mechanism,
float64, whole sequences at a time, nothing cached and nothing shared with muillm_amd/.

A model is a pair (config dict as in config.json, {tensor name: tensor}); `forward` walks it for one
sequence. Every function takes [tokens, features] tensors of one sequence, positions from 0."""

from __future__ import annotations

import math
from typing import Dict, Optional, Tuple

import torch

_HI = torch.float64


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x scaled to unit RMS over the last dimension; eps is added to the mean square."""
    x = x.to(_HI)
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def bigram_rows(tokens: torch.Tensor, buckets: int, mul_prev: int, mul_cur: int) -> torch.Tensor:
    """Row of the bigram table of every token; the first one takes the row behind the buckets."""
    rows = torch.empty_like(tokens)
    rows[0] = buckets
    rows[1:] = (tokens[:-1] * mul_prev + tokens[1:] * mul_cur) % buckets
    return rows


def embed(tokens: torch.Tensor, table: torch.Tensor, scale: float, bigram: Optional[torch.Tensor] = None, buckets: int = 0,
          mul_prev: int = 0, mul_cur: int = 0) -> torch.Tensor:
    x = table.to(_HI)[tokens] * scale
    if bigram is not None:
        x = x + bigram.to(_HI)[bigram_rows(tokens, buckets, mul_prev, mul_cur)]
    return x


def frequencies(dims: int, base: float, scaling: Optional[dict] = None) -> torch.Tensor:
    """[dims / 2] angles per position; scaling: long wavelengths slowed down by `factor`, short ones kept, a
    ramp over original / wavelength between `low` and `high`."""
    f = torch.tensor([float(base) ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=_HI)
    if scaling is None:
        return f
    out = []
    for v in f.tolist():
        length = 2.0 * math.pi / v
        if length < scaling["original"] / scaling["high"]:
            out.append(v)
        elif length > scaling["original"] / scaling["low"]:
            out.append(v / scaling["factor"])
        else:
            s = (scaling["original"] / length - scaling["low"]) / (scaling["high"] - scaling["low"])
            out.append((1.0 - s) * v / scaling["factor"] + s * v)
    return torch.tensor(out, dtype=_HI)


def rotate_pairs(x: torch.Tensor, positions: torch.Tensor, freq: torch.Tensor) -> torch.Tensor:
    """Rotary positions on the first 2 len(freq) of the last dimension of x [tokens, heads, d], pairs (2 i, 2 i + 1)."""
    y = x.to(_HI).clone()
    angle = positions.to(_HI)[:, None, None] * freq
    c, s = torch.cos(angle), torch.sin(angle)
    n = 2 * len(freq)
    u, v = x.to(_HI)[..., 0:n:2], x.to(_HI)[..., 1:n:2]
    y[..., 0:n:2] = u * c - v * s
    y[..., 1:n:2] = v * c + u * s
    return y


def visible(queries: torch.Tensor, keys: torch.Tensor, window: Optional[int], keep_first: int) -> torch.Tensor:
    d = queries[:, None] - keys[None, :]
    if not window:
        return d >= 0
    return (d >= 0) & ((d < window) | (keys[None, :] < keep_first))


def attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, softcap: Optional[float],
              window: Optional[int], keep_first: int, q_start: int = 0) -> torch.Tensor:
    """q [T, H, d] (rotated), k [S, G, d], v [S, G, dv] of positions 0 .. S - 1; query t sits at q_start + t.
    Returns [T, H, dv]."""
    q, k, v = q.to(_HI), k.to(_HI), v.to(_HI)
    t, heads, _ = q.shape
    share = heads // k.shape[1]
    seen = visible(torch.arange(t) + q_start, torch.arange(k.shape[0]), window, keep_first)
    out = torch.empty(t, heads, v.shape[2], dtype=_HI)
    for h in range(heads):
        score = (q[:, h] @ k[:, h // share].T) * scale
        if softcap:
            score = softcap * torch.tanh(score / softcap)
        out[:, h] = torch.softmax(score.masked_fill(~seen, -math.inf), dim=-1) @ v[:, h // share]
    return out


def short_conv(x: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """Causal convolution per channel, x [T, C], taps [C, n] (the last column meets the current token), then silu."""
    x, taps = x.to(_HI), taps.to(_HI)
    n = taps.shape[1]
    padded = torch.cat([torch.zeros(n - 1, x.shape[1], dtype=_HI), x])
    y = sum(padded[j:j + x.shape[0]] * taps[:, j] for j in range(n))
    return y * torch.sigmoid(y)


def unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def channel_delta(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, beta: torch.Tensor, decay: torch.Tensor,
                  state: Optional[torch.Tensor] = None) -> Tuple[torch.Tensor, torch.Tensor]:
    """Delta rule with one decay per key channel, token by token. q, k [T, G, dk], v [T, H, dv], beta [T, H],
    decay [T, H, dk]. Returns (o [T, H, dv], S [H, dk, dv])."""
    t, heads, dv = v.shape
    share = heads // q.shape[1]
    q, k = (x.to(_HI).repeat_interleave(share, dim=1) for x in (q, k))
    s = torch.zeros(heads, q.shape[2], dv, dtype=_HI) if state is None else state.to(_HI).clone()
    out = torch.empty(t, heads, dv, dtype=_HI)
    for p in range(t):
        s = decay[p][:, :, None] * s
        u = beta[p][:, None] * (v[p] - (s * k[p][:, :, None]).sum(1))
        s = s + k[p][:, :, None] * u[:, None, :]
        out[p] = (s * q[p][:, :, None]).sum(1)
    return out, s


def log_decay(h: torch.Tensor, a1: torch.Tensor, a2: torch.Tensor, dt_bias: torch.Tensor, a_log: torch.Tensor) -> torch.Tensor:
    """[T, heads, dk], never positive."""
    z = torch.nn.functional.softplus((h @ a1.to(_HI).T) @ a2.to(_HI).T + dt_bias.to(_HI), threshold=1e9)
    heads = a_log.shape[0]
    return -torch.exp(a_log.to(_HI))[:, None] * z.reshape(h.shape[0], heads, -1)


def dense_mlp(h: torch.Tensor, gate, gate_b, up, up_b, down, down_b) -> torch.Tensor:
    h = h.to(_HI)
    g = h @ gate.to(_HI).T + gate_b.to(_HI)
    return (g * torch.sigmoid(g) * (h @ up.to(_HI).T + up_b.to(_HI))) @ down.to(_HI).T + down_b.to(_HI)


def _attention_layer(x, mx, w, p, eps, plant):
    t = x.shape[0]
    heads, groups, dim, vdim = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = (rms(x @ w[p + "q"].T, eps) * w[p + "q.norm"]).reshape(t, heads, dim)
    k = (rms(x @ w[p + "k"].T, eps) * w[p + "k.norm"]).reshape(t, groups, dim)
    v = (x @ w[p + "v"].T).reshape(t, groups, vdim)
    freq = frequencies(mx["rot"]["dims"], mx["rot"]["base"], mx["rot"].get("scaling"))
    pos = torch.arange(t)
    o = attention(rotate_pairs(q, pos, freq), rotate_pairs(k, pos, freq), v, mx["scale"], mx["softcap"],
                  mx["mask"]["size"] + plant.get("window", 0), mx["mask"]["keep_first"] + plant.get("keep_first", 0))
    return (o.reshape(t, heads * vdim) * torch.sigmoid(x @ w[p + "g"].T)) @ w[p + "o"].T


def _delta_layer(x, mx, w, p, eps):
    t = x.shape[0]
    heads, groups, dim, vdim = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q, k, v = (short_conv(x @ w[p + n].T, w[p + n + ".conv"]) for n in "qkv")
    q = unit(q.reshape(t, groups, dim)) * dim ** -0.5
    k = unit(k.reshape(t, groups, dim))
    beta = torch.sigmoid(x @ w[p + "b"].T)
    decay = torch.exp(log_decay(x, w[p + "a1"], w[p + "a2"], w[p + "dt_bias"], w[p + "A_log"]))
    o, _ = channel_delta(q, k, v.reshape(t, heads, vdim), beta, decay)
    gate = torch.sigmoid((x @ w[p + "g1"].T) @ w[p + "g2"].T)
    return ((rms(o, eps) * w[p + "norm"]).reshape(t, heads * vdim) * gate) @ w[p + "o"].T


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens, plant=None):
    """Logits [T, vocab] and the residual stream after every layer [layers, T, width] of one sequence.
    plant: deliberate mistakes, for tests that show that they would be seen ("window" / "keep_first": added to
    every window / number of kept first tokens)."""
    plant = plant or {}
    w = {k: v.detach().to("cpu", _HI) for k, v in weights.items()}
    eps, m = config["norm"]["eps"], config["residual_mult"]
    e = config["embedding"]
    bg = e.get("bigram")
    tokens = torch.as_tensor(tokens, dtype=torch.int64)
    x = embed(tokens, w["embed"], e["scale"], w.get("bigram"), *((bg["buckets"], bg["mul_prev"], bg["mul_cur"]) if bg else ()))
    stream = []
    for i, layer in enumerate(config["layers"]):
        p = "l%d." % i
        if layer["type"] == "attention":
            y = _attention_layer(x, layer["mixer"], w, p + "mix.", eps, plant)
        elif layer["type"] == "channel_delta":
            y = _delta_layer(x, layer["mixer"], w, p + "mix.", eps)
        else:
            raise ValueError(layer["type"])
        x = x + m * rms(y, eps) * w[p + "norm1"]
        if layer["mlp"] is not None:
            y = dense_mlp(x, *(w[p + "mlp." + n] for n in ("gate", "gate.b", "up", "up.b", "down", "down.b")))
            x = x + m * rms(y, eps) * w[p + "norm2"]
        stream.append(x)
    return ((rms(x, eps) * w["final.norm"]) @ w["head"].T) * config["logit_scale"], torch.stack(stream)
