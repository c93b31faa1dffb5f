"""CPU restatement of the Salepel decoder (test infrastructure only): one function per mechanism,
float64, whole sequences at a time, nothing cached and nothing shared with muillm_amd/.

A model is a pair (config dict as in config.json, {tensor name: tensor}); `forward` walks it for one
sequence. Every function takes [tokens, features] tensors of one sequence, positions from 0."""

from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

_HI = torch.float64


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x scaled to unit RMS over the last dimension; eps is added to the mean square."""
    x = x.to(_HI)
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rotate(x: torch.Tensor, positions: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """Rotary positions on the first `dims` of the last dimension, x [tokens, ..., d], pairs (i, i + dims/2)."""
    x = x.to(_HI)
    half = dims // 2
    freq = float(base) ** (-2.0 * torch.arange(half, dtype=_HI) / dims)
    angle = positions.to(_HI).reshape([-1] + [1] * (x.dim() - 1)) * freq
    u, v = x[..., :half], x[..., half:dims]
    c, s = torch.cos(angle), torch.sin(angle)
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], dim=-1)


def latent_rows(h: torch.Tensor, w_dkv: torch.Tensor, gain: torch.Tensor, kv_rank: int, rot_dim: int, base: float,
                eps: float, start: int = 0) -> Tuple[torch.Tensor, torch.Tensor]:
    """(latent c [T, kv_rank], rotated key part [T, rot_dim]) of tokens start, start + 1, ..."""
    y = h.to(_HI) @ w_dkv.to(_HI).T
    c = rms(y[:, :kv_rank], eps) * gain.to(_HI)
    return c, rotate(y[:, kv_rank:], torch.arange(start, start + h.shape[0]), rot_dim, base)


def latent_attention(q: torch.Tensor, c: torch.Tensor, k_rot: torch.Tensor, w_uk: torch.Tensor, w_uv: torch.Tensor,
                     heads: int, dim: int, rot_dim: int, vdim: int, scale: float, window: Optional[int],
                     q_start: int = 0) -> torch.Tensor:
    """q [T, heads, dim + rot_dim] (rotated), c / k_rot of positions 0..S-1; query t sits at q_start + t and
    sees positions p - window + 1 .. p. Returns [T, heads * vdim]."""
    q, c, k_rot = q.to(_HI), c.to(_HI), k_rot.to(_HI)
    t, s = q.shape[0], c.shape[0]
    k = (c @ w_uk.to(_HI).T).reshape(s, heads, dim)
    v = (c @ w_uv.to(_HI).T).reshape(s, heads, vdim)
    d = (torch.arange(t) + q_start)[:, None] - torch.arange(s)[None, :]
    seen = d >= 0
    if window:
        seen &= d < window
    out = torch.empty(t, heads, vdim, dtype=_HI)
    for h in range(heads):
        score = (q[:, h, :dim] @ k[:, h].T + q[:, h, dim:] @ k_rot.T) * scale
        out[:, h] = torch.softmax(score.masked_fill(~seen, -math.inf), dim=-1) @ v[:, h]
    return out.reshape(t, heads * vdim)


def mlstm(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, i_pre: torch.Tensor, f_pre: torch.Tensor, cap: float,
          state=None):
    """Matrix memory, token by token. q, k [T, H, dk] (already scaled), v [T, H, dv]; i_pre, f_pre [T, H]
    gate pre-activations with their biases. Returns (o [T, H, dv], (S, n, m))."""
    q, k, v = q.to(_HI), k.to(_HI), v.to(_HI)
    t, heads, dk = q.shape
    dv = v.shape[2]
    log_i = cap * torch.tanh(i_pre.to(_HI) / cap)
    log_f = torch.nn.functional.logsigmoid(cap * torch.tanh(f_pre.to(_HI) / cap))
    if state is None:
        big, n, m = torch.zeros(heads, dk, dv, dtype=_HI), torch.zeros(heads, dk, dtype=_HI), torch.zeros(heads, dtype=_HI)
    else:
        big, n, m = (s.clone() for s in state)
    out = torch.empty(t, heads, dv, dtype=_HI)
    for p in range(t):
        m_new = torch.maximum(log_f[p] + m, log_i[p])
        keep, add = torch.exp(log_f[p] + m - m_new), torch.exp(log_i[p] - m_new)
        big = keep[:, None, None] * big + add[:, None, None] * k[p][:, :, None] * v[p][:, None, :]
        n = keep[:, None] * n + add[:, None] * k[p]
        m = m_new
        den = torch.maximum((n * q[p]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out[p] = (big * q[p][:, :, None]).sum(1) / den[:, None]
    return out, (big, n, m)


def router(h: torch.Tensor, w: torch.Tensor, correction: torch.Tensor, top: int) -> Tuple[torch.Tensor, torch.Tensor]:
    """(chosen experts [T, top], their weights): chosen by softmax + correction, weighted by softmax alone."""
    s = torch.softmax(h.to(_HI) @ w.to(_HI).T, dim=-1)
    chosen = torch.topk(s + correction.to(_HI), top, dim=-1).indices
    return chosen, s.gather(-1, chosen)


def expert(h: torch.Tensor, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor, limit: float) -> torch.Tensor:
    h = h.to(_HI)
    g = (h @ gate.to(_HI).T).clamp(max=limit)
    u = (h @ up.to(_HI).T).clamp(min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ down.to(_HI).T


def moe(h: torch.Tensor, router_w, correction, experts: List[Tuple[torch.Tensor, torch.Tensor, torch.Tensor]], top: int,
        limit: float) -> torch.Tensor:
    """Weighted sum over the chosen experts; router outputs beyond len(experts) return h itself."""
    h = h.to(_HI)
    chosen, weight = router(h, router_w, correction, top)
    out = torch.zeros_like(h)
    for e in range(router_w.shape[0]):
        share = torch.where(chosen == e, weight, torch.zeros_like(weight)).sum(-1)
        rows = (chosen == e).any(-1).nonzero().flatten()
        if rows.numel():
            y = expert(h[rows], *experts[e], limit) if e < len(experts) else h[rows]
            out[rows] += share[rows, None] * y
    return out


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens, plant=None):
    """Logits [T, vocab] and the residual stream after every layer [layers, T, width] of one sequence.
    plant: deliberate mistakes, for tests that show that they would be seen ("window": added to every window)."""
    plant = plant or {}
    w = {k: v.detach().to("cpu", _HI) for k, v in weights.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.int64)] * config["embedding"]["scale"]
    t = x.shape[0]
    pos = torch.arange(t)
    rows, stream = {}, []
    for li, layer in enumerate(config["layers"]):
        p = "l%d." % li
        mx = layer["mixer"]
        h = rms(x, eps) * w[p + "norm1"]
        if layer["type"] == "latent_attention":
            heads, dim, rd, vd, kr = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
            base = mx["rot"]["base"]
            cq = rms(h @ w[p + "mix.dq"].T, eps) * w[p + "mix.dq.norm"]
            q = (cq @ w[p + "mix.uq"].T).reshape(t, heads, dim + rd)
            q = torch.cat([q[..., :dim], rotate(q[..., dim:], pos, rd, base)], dim=-1)
            if "kv_from" in mx:
                src = mx["kv_from"]
            else:
                src = li
                rows[li] = latent_rows(h, w[p + "mix.dkv"], w[p + "mix.dkv.norm"], kr, rd, base, eps)
            c, kr_rot = rows[src]
            o = latent_attention(q, c, kr_rot, w[p + "mix.uk"], w[p + "mix.uv"], heads, dim, rd, vd, mx["scale"],
                                 mx["mask"]["size"] + plant.get("window", 0))
            y = o @ w[p + "mix.o"].T
        elif layer["type"] == "mlstm":
            heads, dk, dv = mx["heads"], mx["dim"], mx["vdim"]
            q = (h @ w[p + "mix.q"].T).reshape(t, heads, dk) * dk ** -0.5
            k = (h @ w[p + "mix.k"].T).reshape(t, heads, dk)
            v = (h @ w[p + "mix.v"].T).reshape(t, heads, dv)
            o, _ = mlstm(q, k, v, h @ w[p + "mix.i"].T + w[p + "mix.i.b"], h @ w[p + "mix.f"].T + w[p + "mix.f.b"],
                         mx["gate_cap"])
            o = rms(o, eps).reshape(t, heads * dv) * w[p + "mix.norm"] * torch.sigmoid(h @ w[p + "mix.g"].T)
            y = o @ w[p + "mix.o"].T
        else:
            raise ValueError(layer["type"])
        x = x + rms(y, eps) * w[p + "norm1b"]
        ff = layer["mlp"]
        if ff is not None:
            h = rms(x, eps) * w[p + "norm2"]
            experts = [tuple(w["%smlp.e%d.%s" % (p, e, n)] for n in ("gate", "up", "down"))
                       for e in range(ff["router"]["experts"])]
            y = moe(h, w[p + "mlp.router"], w[p + "mlp.correction"], experts, ff["router"]["top"], ff["expert"]["limit"])
            x = x + rms(y, eps) * w[p + "norm2b"]
        stream.append(x)
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T, torch.stack(stream)
