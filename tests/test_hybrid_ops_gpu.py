"""The mechanisms of hybrid decoders, one by one, against the float64 oracle: residual / norm boundary,
32-bit linears, routing, experts, latent attention (all routes), matrix-memory recurrence (step by step and
in chunks)."""
import math

import pytest
import torch

from muillm_amd import _lib, hybrid_ops as ops
from oracle import salepel as oracle

pytestmark = pytest.mark.gpu
DEV = "cuda"
DTYPES = [torch.float32, torch.bfloat16, torch.float16]
# relative to the largest reference value
REL = {torch.float32: 2e-5, torch.bfloat16: 1.5e-2, torch.float16: 2e-3}


def _rand(g, *shape, std=1.0):
    return torch.randn(*shape, generator=g) * std


def _close(got, ref, rel, what=""):
    got, ref = got.detach().to("cpu", torch.float64), ref.to(torch.float64)
    assert got.shape == ref.shape, (what, got.shape, ref.shape)
    assert bool(torch.isfinite(got).all()), what
    err = float((got - ref).abs().max() / ref.abs().max().clamp_min(1e-30))
    assert err <= rel, f"{what}: {err:.2e} > {rel:.1e}"


# --------------------------------------------------------------------------------------
# residual / norm
# --------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,k", [(1, 96), (3, 37), (5, 2056), (2, 5000), (2, 16384), (1, 20008)])
def test_residual_norm(dtype, rows, k):
    g = torch.Generator().manual_seed(k)
    x, y = _rand(g, rows, k), _rand(g, rows, k, std=3.0).to(dtype)
    pg, ng = (1 + 0.2 * _rand(g, k)).to(dtype), (1 + 0.2 * _rand(g, k)).to(dtype)
    eps = 0.1  # large enough to show where it is added
    ref_x = x.double() + oracle.rms(y, eps) * pg.double()
    out, h = ops.residual_norm(x.to(DEV), y.to(DEV), pg.to(DEV), ng.to(DEV), eps)
    _close(out, ref_x, 3e-6, "residual")
    _close(h, oracle.rms(ref_x, eps) * ng.double(), max(REL[dtype] / 3, 3e-6), "norm")
    # no post norm, no residual, a scale (the embedding), no following norm
    out, h = ops.residual_norm(None, y.to(DEV), None, None, eps, y_scale=5.5)
    assert h is None
    _close(out, 5.5 * y.double(), 1e-6)
    out, h = ops.residual_norm(x.to(DEV), y.to(DEV), pg.to(DEV), None, eps)
    _close(out, ref_x, 3e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [72, 77])
def test_moe_residual_norm(dtype, width):
    g = torch.Generator().manual_seed(1)
    tokens, top, n_exp = 5, 3, 4
    pairs, ident = _rand(g, tokens * top, width).to(dtype), _rand(g, tokens, width).to(dtype)
    expert = torch.tensor([[0, 5, 3], [4, 5, 6], [1, 2, 0], [3, 4, 1], [2, 0, 6]], dtype=torch.int32)
    weight = torch.rand(tokens, top, generator=g)
    pairs[(expert.reshape(-1) >= n_exp)] = float("nan")  # rows of identity experts are never written, nor read
    ref = torch.zeros(tokens, width, dtype=torch.float64)
    for t in range(tokens):
        for j in range(top):
            src = pairs[t * top + j] if expert[t, j] < n_exp else ident[t]
            ref[t] += weight[t, j].double() * src.double()
    out = ops.MoEOutput(pairs.to(DEV), ident.to(DEV), expert.to(DEV), weight.to(DEV), n_exp)
    _close(out.dense(), ref, 2e-6)
    x, gain = _rand(g, tokens, width), (1 + 0.1 * _rand(g, width)).to(dtype)
    rx = x.double() + oracle.rms(ref, 1e-3) * gain.double()
    o, h = ops.residual_norm(x.to(DEV), out, gain.to(DEV), gain.to(DEV), 1e-3)
    _close(o, rx, 3e-6)
    _close(h, oracle.rms(rx, 1e-3) * gain.double(), max(REL[dtype] / 3, 3e-6))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("tokens,n,k", [(1, 7, 96), (3, 6, 250), (16, 33, 40), (17, 5, 72), (130, 70, 1096), (18, 4, 51)])
def test_linear_f32(dtype, tokens, n, k):
    g = torch.Generator().manual_seed(tokens)
    x, w, b = _rand(g, tokens, k).to(dtype), _rand(g, n, k).to(dtype), _rand(g, n).to(dtype)
    y = ops.linear_f32(x.to(DEV), w.to(DEV), b.to(DEV))
    assert y.dtype == torch.float32
    _close(y, x.double() @ w.double().T + b.double(), 3e-6)
    _close(ops.linear_f32(x.to(DEV), w.to(DEV)), x.double() @ w.double().T, 3e-6)


# --------------------------------------------------------------------------------------
# mixture of experts
# --------------------------------------------------------------------------------------
@pytest.mark.parametrize("tokens,experts,identity,top", [(1, 5, 2, 3), (7, 1, 0, 1), (40, 70, 60, 9), (100, 6, 3, 9), (300, 12, 1, 2),
                                                         (9, 200, 0, 1)])
@pytest.mark.parametrize("tile", [0, 16, 128, 256])
def test_route(tokens, experts, identity, top, tile):
    g = torch.Generator().manual_seed(tokens)
    n = experts + identity
    logits, corr = _rand(g, tokens, n, std=2.0), _rand(g, n, std=0.05)
    expert, weight, pairs, tiles = ops.moe_route(logits.to(DEV), corr.to(DEV), experts, top, tile)
    s = torch.softmax(logits.double(), -1)
    order = torch.topk(s + corr.double(), top, dim=-1).indices
    assert torch.equal(expert.cpu().long().sort(-1).values, order.sort(-1).values)
    _close(weight, s.gather(-1, expert.cpu().long()), 2e-6)
    if not tile:
        return
    real = (expert.cpu().reshape(-1) < experts)
    tiles, pairs, flat = tiles.cpu(), pairs.cpu().long(), expert.cpu().reshape(-1)
    seen, n_tiles = [], int(tiles[0, 2])
    for e, first, count, _ in tiles[1:1 + n_tiles].tolist():
        assert 1 <= count <= tile
        part = pairs[first:first + count]
        assert bool((flat[part] == e).all())
        seen += part.tolist()
    assert sorted(seen) == real.nonzero().flatten().tolist()
    assert bool((tiles[1 + n_tiles:, 2] == 0).all())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("tokens,experts,identity,top,width,ff", [
    (1, 5, 2, 3, 96, 56), (2, 3, 0, 3, 64, 40), (16, 4, 1, 2, 200, 128), (33, 9, 4, 4, 96, 24), (150, 3, 2, 4, 128, 192),
    (401, 3, 1, 2, 96, 72), (620, 2, 1, 2, 128, 200), (5, 4, 1, 2, 51, 23), (90, 1, 0, 1, 64, 64)])
def test_experts(dtype, tokens, experts, identity, top, width, ff):
    g = torch.Generator().manual_seed(tokens + width)
    x, limit = _rand(g, tokens, width).to(dtype), 0.6  # clamps in most of the places
    gate, up = _rand(g, experts, ff, width, std=width ** -0.5).to(dtype), _rand(g, experts, ff, width, std=width ** -0.5).to(dtype)
    down = _rand(g, experts, width, ff, std=ff ** -0.5).to(dtype)
    rw, corr = _rand(g, experts + identity, width, std=2 * width ** -0.5).to(dtype), _rand(g, experts + identity, std=0.02).to(dtype)
    tile = ops.moe_tile_pairs(dtype, tokens, top, experts, width, ff)
    logits = ops.linear_f32(x.to(DEV), rw.to(DEV))
    expert, weight, pairs, tiles = ops.moe_route(logits, corr.to(DEV), experts, top, tile)
    out = ops.moe_experts(x.to(DEV), gate.to(DEV), up.to(DEV), down.to(DEV), limit, expert, pairs, tiles, tile)
    e = expert.cpu().reshape(-1)
    for i in range(experts):
        rows = (e == i).nonzero().flatten()
        if rows.numel():
            _close(out[rows.to(DEV)], oracle.expert(x[rows // top], gate[i], up[i], down[i], limit), REL[dtype], f"expert {i}")
    y = ops.MoEOutput(out, x.to(DEV), expert, weight, experts).dense()
    ref = oracle.moe(x, rw, corr, [(gate[i], up[i], down[i]) for i in range(experts)], top, limit)
    _close(y, ref, REL[dtype], "sum")


def test_experts_of_every_tile_size_agree():
    """The same pairs through tiles of every width (bf16)."""
    g = torch.Generator().manual_seed(3)
    tokens, experts, top, width, ff, dtype = 200, 3, 2, 160, 96, torch.bfloat16
    x = _rand(g, tokens, width).to(dtype).to(DEV)
    gate, up = (_rand(g, experts, ff, width, std=0.1).to(dtype).to(DEV) for _ in range(2))
    down = _rand(g, experts, width, ff, std=0.1).to(dtype).to(DEV)
    logits = _rand(g, tokens, experts).to(DEV)
    outs = []
    for tile in (16, 128, 256):
        expert, _, pairs, tiles = ops.moe_route(logits, torch.zeros(experts, dtype=dtype, device=DEV), experts, top, tile)
        outs.append(ops.moe_experts(x, gate, up, down, 1.0, expert, pairs, tiles, tile).float())
    _close(outs[1], outs[0].cpu(), 1e-2)
    _close(outs[2], outs[0].cpu(), 1e-2)


# --------------------------------------------------------------------------------------
# latent attention
# --------------------------------------------------------------------------------------
def _latent_case(seed, dtype, s, t, heads, dim, rot, vdim, kv_rank, std=1.0):
    g = torch.Generator().manual_seed(seed)
    c, r = _rand(g, s, kv_rank).to(dtype), _rand(g, s, rot).to(dtype)
    q = _rand(g, t, heads * (dim + rot), std=std).to(dtype)
    uk, uv = _rand(g, heads * dim, kv_rank, std=kv_rank ** -0.5).to(dtype), _rand(g, heads * vdim, kv_rank, std=kv_rank ** -0.5).to(dtype)
    return c, r, q, uk, uv


def _cos_sin(pos, rot, base):
    f = float(base) ** (-2.0 * torch.arange(rot // 2, dtype=torch.float64) / rot)
    a = pos.double()[:, None] * f
    return torch.cat([a.cos(), a.sin()], -1).float().to(DEV)


def _attend(dtype, c, r, q, uk, uv, heads, dim, vdim, scale, window, q_first, base, route, row_start=None, batch=1, capacity=None):
    """Through the library: caches of `capacity` rows whose unused rows hold huge values."""
    s, t, rot = c.shape[0], q.shape[0], r.shape[1]
    cap = capacity or s + 7
    cc = torch.full((batch, cap, c.shape[1]), 1e4, dtype=dtype, device=DEV)
    rc = torch.full((batch, cap, rot), 1e4, dtype=dtype, device=DEV)
    cc[:, :s], rc[:, :s] = c.to(DEV), r.to(DEV)
    pos = torch.arange(q_first, q_first + t)
    cs = torch.cat([_cos_sin(pos - (0 if row_start is None else int(row_start[i])), rot, base) for i in range(batch)])
    qq = q.to(DEV)[None].repeat(batch, 1, 1)
    rs = None if row_start is None else row_start.to(DEV)
    if route == _lib.MUI_LATENT_PREFILL:
        first = max(0, q_first - window + 1) if window else 0
        kv = [torch.cat([cc[i, first:s] @ uk.to(DEV).T, cc[i, first:s] @ uv.to(DEV).T], -1).contiguous() for i in range(batch)]
        return ops.latent_prefill_attention(qq, cs, kv, first, rc, rs, q_first, heads, dim, vdim, scale, window)
    return ops.latent_attention(qq, cs, uk.to(DEV), uv.to(DEV), cc, rc, pos.to(DEV), rs, heads, dim, vdim, scale, window, route)


def _attend_oracle(c, r, q, uk, uv, heads, dim, vdim, scale, window, q_first, base, row_start=0):
    rot, t = r.shape[1], q.shape[0]
    qh = q.double().reshape(t, heads, dim + rot)
    qr = oracle.rotate(qh[..., dim:], torch.arange(q_first, q_first + t) - row_start, rot, base)
    return oracle.latent_attention(torch.cat([qh[..., :dim], qr], -1), c[row_start:], r[row_start:], uk, uv, heads, dim, rot, vdim,
                                   scale, window or None, q_first - row_start)


ROUTES = {"plain": _lib.MUI_LATENT_PLAIN, "decode": _lib.MUI_LATENT_DECODE, "prefill": _lib.MUI_LATENT_PREFILL}
SIZES = [(3, 24, 8, 40, 48), (1, 16, 2, 8, 8), (17, 40, 24, 32, 136), (5, 96, 32, 72, 264), (2, 128, 64, 128, 512), (4, 160, 64, 200, 72),
         (2, 20, 6, 12, 24)]


@pytest.mark.parametrize("dtype,route", [(torch.float32, "plain"), (torch.bfloat16, "plain"), (torch.bfloat16, "decode"),
                                         (torch.bfloat16, "prefill"), (torch.float16, "decode"), (torch.float16, "prefill")])
@pytest.mark.parametrize("heads,dim,rot,vdim,kv_rank", SIZES)
def test_latent_attention_routes(dtype, route, heads, dim, rot, vdim, kv_rank):
    for t, q_first, window in ((1, 0, 5), (1, 200, 0), (1, 200, 130), (2, 63, 64), (5, 190, 33), (20, 0, 9), (150, 90, 70), (131, 0, 0)):
        if route == "decode" and t > 20:
            continue
        case = _latent_case(t + q_first, dtype, q_first + t, t, heads, dim, rot, vdim, kv_rank)
        args = (heads, dim, vdim, (dim + rot) ** -0.5, window, q_first, 700.0)
        got = _attend(dtype, *case, *args, ROUTES[route])[0]
        _close(got, _attend_oracle(*case, *args), REL[dtype], f"t={t} first={q_first} window={window}")


@pytest.mark.parametrize("dtype,route", [(torch.float32, "plain"), (torch.bfloat16, "decode"), (torch.bfloat16, "prefill")])
@pytest.mark.parametrize("window", [1, 2, 63, 64, 65, 129])
def test_latent_attention_window_edge(dtype, route, window):
    """One key stands out by far: the query that just sees it takes (almost) only its value, the next one
    does not see it at all."""
    heads, dim, rot, vdim, kv_rank, hot = 2, 16, 8, 16, 32, 70
    s = hot + window + 30
    g = torch.Generator().manual_seed(window)
    c, r = _rand(g, s, kv_rank, std=0.1).to(dtype), _rand(g, s, rot, std=0.1).to(dtype)
    uk, uv = _rand(g, heads * dim, kv_rank).to(dtype), _rand(g, heads * vdim, kv_rank).to(dtype)
    c[hot] = 4 * torch.sign(_rand(g, kv_rank)).to(dtype)
    khot = (c[hot].double() @ uk.double().T).reshape(heads, dim)
    base = 50.0
    queries = [hot, hot + window - 1, hot + window, hot + window + 1]  # own, last to see it, first two not to
    for t in sorted({1, 25, min(window + 20, 140)}):
        for p in queries:
            first = max(0, p - t + 1) if route == "prefill" else p
            n = p - first + 1
            q = torch.zeros(n, heads, dim + rot, dtype=torch.float64)
            q[..., :dim] = khot
            q = q.reshape(n, -1).to(dtype)
            args = (heads, dim, vdim, 0.05, window, first, base)
            got = _attend(dtype, c[:p + 1], r[:p + 1], q, uk, uv, *args, ROUTES[route])[0]
            ref = _attend_oracle(c[:p + 1], r[:p + 1], q, uk, uv, *args)
            _close(got[-1:], ref[-1:], REL[dtype], f"window={window} query={p - hot} t={t}")
            hot_value = (c[hot].double() @ uv.double().T)
            share = float((got[-1].cpu().double() - hot_value).abs().max() / hot_value.abs().max())
            assert (share < 0.02) == (p - hot < window), (window, p - hot, share)


@pytest.mark.parametrize("route", ["decode", "prefill", "plain"])
def test_latent_attention_batch_rows_and_left_padding(route):
    dtype, heads, dim, rot, vdim, kv_rank, window = torch.bfloat16, 3, 24, 8, 40, 48, 33
    t, q_first = (2, 80) if route == "decode" else (70, 10)
    c, r, q, uk, uv = _latent_case(5, dtype, q_first + t, t, heads, dim, rot, vdim, kv_rank)
    starts = torch.tensor([0, 60 if route == "decode" else 5, q_first + t - 1])
    args = (heads, dim, vdim, 0.2, window, q_first, 300.0)
    got = _attend(dtype, c, r, q, uk, uv, *args, ROUTES[route], row_start=starts, batch=3)
    for i, st in enumerate(starts.tolist()):
        live = torch.arange(q_first, q_first + t) >= st
        skip = max(0, st - q_first)
        a = (heads, dim, vdim, 0.2, window, q_first + skip, 300.0)
        ref = _attend_oracle(c, r, q[skip:], uk, uv, *a, row_start=st)
        _close(got[i].cpu()[live], ref, REL[dtype], f"row {i}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_latent_prepare(dtype):
    g = torch.Generator().manual_seed(2)
    b, t, q_rank, kv_rank, rot, cap, eps, base = 2, 3, 56, 48, 10, 300000, 0.05, 10000.0
    down = _rand(g, b, t, q_rank + kv_rank + rot).to(dtype)
    qg, kg = (1 + 0.2 * _rand(g, q_rank)).to(dtype), (1 + 0.2 * _rand(g, kv_rank)).to(dtype)
    inv = base ** (-2.0 * torch.arange(rot // 2, dtype=torch.float64) / rot)
    for slot in (0, 63, 262143):  # far positions: the angle is reduced before it is rounded
        cc, rc = torch.zeros(b, cap, kv_rank, dtype=dtype, device=DEV), torch.zeros(b, cap, rot, dtype=dtype, device=DEV)
        pos = torch.arange(slot, slot + t)
        ql, cs = ops.latent_prepare(down.to(DEV), qg.to(DEV), kg.to(DEV), eps, inv.to(DEV), pos.to(DEV), None, cc, rc)
        _close(ql, oracle.rms(down[..., :q_rank], eps) * qg.double(), REL[dtype] / 2)
        for i in range(b):
            _close(cc[i, slot:slot + t], oracle.rms(down[i, :, q_rank:q_rank + kv_rank], eps) * kg.double(), REL[dtype] / 2)
            _close(rc[i, slot:slot + t], oracle.rotate(down[i, :, q_rank + kv_rank:], pos, rot, base), REL[dtype] / 2)
        angle = pos.double()[:, None] * inv
        _close(cs[:t], torch.cat([angle.cos(), angle.sin()], -1), 1e-6)
        assert float(cc[:, slot + t:].abs().max()) == 0 and (slot == 0 or float(cc[:, :slot].abs().max()) == 0)
    # a layer without rows of its own leaves the caches alone; slots outside the cache are skipped
    cc, rc = torch.zeros(b, 4, kv_rank, dtype=dtype, device=DEV), torch.zeros(b, 4, rot, dtype=dtype, device=DEV)
    ops.latent_prepare(down[..., :q_rank].contiguous().to(DEV), qg.to(DEV), None, eps, inv.to(DEV), torch.arange(3).to(DEV), None, cc, rc)
    assert float(cc.abs().max()) == 0
    ops.latent_prepare(down.to(DEV), qg.to(DEV), kg.to(DEV), eps, inv.to(DEV), torch.arange(2, 5).to(DEV), None, cc, rc)
    assert float(cc[:, :2].abs().max()) == 0 and float(cc[:, 3].abs().max()) > 0


# --------------------------------------------------------------------------------------
# matrix memory
# --------------------------------------------------------------------------------------
def _mlstm_case(seed, dtype, b, t, heads, dk, dv, f_bias=3.0, gate_std=2.0):
    g = torch.Generator().manual_seed(seed)
    proj = _rand(g, b, t, heads * (2 * dk + 2 * dv)).to(dtype)
    gates = _rand(g, b, t, 2 * heads, std=gate_std)
    gates[..., heads:] += f_bias
    return proj, gates


def _mlstm_run(proj, gates, heads, dk, dv, cap, cuts, row_start=None, state=None):
    """In portions `cuts`; returns o and the state."""
    b, t = proj.shape[0], proj.shape[1]
    slices = ops.mlstm_slices(dv)
    if state is None:
        state = (torch.zeros(b, heads, dk, dv, device=DEV), torch.zeros(b, heads, slices, dk, device=DEV),
                 torch.zeros(b, heads, slices, device=DEV))
    outs, at = [], 0
    for n in cuts:
        p = proj[:, at:at + n].contiguous().to(DEV)
        q, k, v = p[..., :heads * dk], p[..., heads * dk:2 * heads * dk], p[..., 2 * heads * dk:heads * (2 * dk + dv)]
        outs.append(ops.mlstm(q, k, v, gates[:, at:at + n].contiguous().to(DEV), state, dk ** -0.5, cap,
                              torch.arange(at, at + n, device=DEV), row_start, heads))
        at += n
    assert at == t
    return torch.cat(outs, 1), state


def _mlstm_oracle(proj, gates, heads, dk, dv, cap):
    t = proj.shape[0]
    p = proj.double()
    q = p[:, :heads * dk].reshape(t, heads, dk) * dk ** -0.5
    k = p[:, heads * dk:2 * heads * dk].reshape(t, heads, dk)
    v = p[:, 2 * heads * dk:heads * (2 * dk + dv)].reshape(t, heads, dv)
    return oracle.mlstm(q, k, v, gates[:, :heads], gates[:, heads:], cap)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dk,dv", [(2, 40, 72), (3, 24, 20), (1, 5, 7), (4, 64, 64), (2, 130, 66), (1, 288, 33)])
def test_mlstm_step_and_chunks(dtype, heads, dk, dv):
    t, cap = 210, 7.0
    proj, gates = _mlstm_case(dk, dtype, 1, t, heads, dk, dv)
    ref, (rs, rn, rm) = _mlstm_oracle(proj[0], gates[0], heads, dk, dv, cap)
    for cuts in ([t], [2] * 105, [1] * 20 + [190], [64, 64, 64, 18], [17, 2, 63, 65, 3, 60], [100, 1, 1, 108]):
        o, (s, n, m) = _mlstm_run(proj, gates, heads, dk, dv, cap, cuts)
        _close(o[0], ref, 5e-5, f"{cuts[:6]}")
        _close(s[0], rs, 2e-5)
        for sl in range(n.shape[2]):
            _close(n[0, :, sl], rn, 2e-5)
            _close(m[0, :, sl], rm, 2e-5)


@pytest.mark.parametrize("f_bias,gate_std,cap", [(-20.0, 1.0, 15.0), (0.0, 30.0, 15.0), (0.0, 0.0, 3.0), (9.0, 4.0, 1.0)])
def test_mlstm_gate_regimes(f_bias, gate_std, cap):
    """Closed forget gates (sums over a chunk reach hundreds), saturated caps, constant gates."""
    heads, dk, dv, t = 2, 32, 48, 300
    proj, gates = _mlstm_case(9, torch.float32, 1, t, heads, dk, dv, f_bias, gate_std)
    ref, _ = _mlstm_oracle(proj[0], gates[0], heads, dk, dv, cap)
    for cuts in ([t], [1] * 40 + [260], [150, 2, 148]):
        o, _ = _mlstm_run(proj, gates, heads, dk, dv, cap, cuts)
        _close(o[0], ref, 3e-4, f"{cuts[:3]}")


def test_mlstm_denominator_floor():
    """n . q near zero: the output is divided by e^-m plus the constant, and m starts at 0 (closed input
    gates do not drag it below what the forget gate leaves)."""
    heads, dk, dv, t = 1, 8, 8, 80
    proj, gates = _mlstm_case(4, torch.float32, 1, t, heads, dk, dv)
    proj[..., :dk] *= 1e-3
    gates[..., 0] = -6.0
    ref, _ = _mlstm_oracle(proj[0], gates[0], heads, dk, dv, 15.0)
    for cuts in ([t], [1] * t):
        o, _ = _mlstm_run(proj, gates, heads, dk, dv, 15.0, cuts)
        _close(o[0], ref, 2e-5)


def test_mlstm_batch_and_left_padding():
    heads, dk, dv, t = 2, 40, 72, 150
    proj, gates = _mlstm_case(8, torch.bfloat16, 3, t, heads, dk, dv)
    starts = torch.tensor([0, 70, 3])
    for cuts in ([t], [2, 148], [1] * 5 + [145]):
        o, (s, _, _) = _mlstm_run(proj, gates, heads, dk, dv, 9.0, cuts, row_start=starts.to(DEV))
        for i, st in enumerate(starts.tolist()):
            ref, (rs, _, _) = _mlstm_oracle(proj[i, st:], gates[i, st:], heads, dk, dv, 9.0)
            _close(o[i, st:], ref, 2e-5, f"row {i}")
            _close(s[i], rs, 2e-5)


def test_mlstm_long_prompt_in_segments(monkeypatch):
    heads, dk, dv, t = 1, 16, 24, 500
    proj, gates = _mlstm_case(6, torch.float32, 2, t, heads, dk, dv, f_bias=6.0)
    monkeypatch.setattr(ops, "MLSTM_SEGMENT", 128)
    o, _ = _mlstm_run(proj, gates, heads, dk, dv, 9.0, [t])
    for i in range(2):
        ref, _ = _mlstm_oracle(proj[i], gates[i], heads, dk, dv, 9.0)
        _close(o[i], ref, 2e-5)


@pytest.mark.parametrize("dtype", DTYPES)
def test_mlstm_output(dtype):
    g = torch.Generator().manual_seed(1)
    b, t, heads, dv = 2, 5, 3, 70
    o, gain = _rand(g, b, t, heads, dv), (1 + 0.2 * _rand(g, heads * dv)).to(dtype)
    proj = _rand(g, b, t, 50 + heads * dv).to(dtype)
    y = ops.mlstm_output(o.to(DEV), gain.to(DEV), proj.to(DEV)[..., 50:], 0.02)
    ref = oracle.rms(o, 0.02).reshape(b, t, -1) * gain.double() * torch.sigmoid(proj[..., 50:].double())
    _close(y, ref, REL[dtype] / 2 if dtype != torch.float32 else 3e-6)


def test_operands_are_checked():
    x = torch.zeros(2, 8, device=DEV, dtype=torch.bfloat16)
    with pytest.raises(RuntimeError):
        ops.residual_norm(None, x, torch.ones(7, device=DEV, dtype=torch.bfloat16), None, 1e-5)
    with pytest.raises(RuntimeError):
        ops.linear_f32(x, torch.zeros(3, 9, device=DEV, dtype=torch.bfloat16))
    with pytest.raises(ValueError):
        ops.residual_norm(None, x.to(torch.float64), None, None, 1e-5)
    assert math.isfinite(float(ops.residual_norm(None, x, None, None, 1e-5)[0].sum()))
