"""The mechanisms of the Zufadra decoder, one by one, against the float64 oracle: scaled branches, biased gate/up products,
bigram embedding, query / key preparation, windowed attention with sinks (all routes), the gated delta rule (step by step,
in chunks, cut anywhere)."""
import math

import pytest
import torch

from muillm_amd import _lib, hybrid_ops as ops, muillm_ext
from oracle import zufadra as oracle

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


def _slots(start, n):
    return torch.arange(start, start + n, device=DEV)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,k", [(1, 104), (3, 37), (5, 2056)])
def test_scaled_branch_and_plain_input(dtype, rows, k):
    g = torch.Generator().manual_seed(k)
    x, y = _rand(g, rows, k), _rand(g, rows, k, std=3.0).to(dtype)
    pg, ng = (1 + 0.2 * _rand(g, k)).to(dtype), (1 + 0.2 * _rand(g, k)).to(dtype)
    ref = x.double() + 0.6 * oracle.rms(y, 0.1) * pg.double()
    out, h = ops.residual_norm(x.to(DEV), y.to(DEV), pg.to(DEV), None, 0.1, branch_scale=0.6, emit=True)
    _close(out, ref, 3e-6)
    _close(h, ref, max(REL[dtype] / 3, 3e-6))
    out, h = ops.residual_norm(x.to(DEV), y.to(DEV), pg.to(DEV), ng.to(DEV), 0.1, branch_scale=0.6, next_scale=0.3)
    _close(out, ref, 3e-6)
    _close(h, 0.3 * oracle.rms(ref, 0.1) * ng.double(), max(REL[dtype] / 3, 3e-6))
    out, h = ops.residual_norm(None, y.to(DEV), None, None, 0.0, y_scale=1.5, emit=True)
    _close(out, 1.5 * y.double(), 1e-6)
    _close(h, 1.5 * y.double(), max(REL[dtype] / 3, 1e-6))


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float16])
@pytest.mark.parametrize("k,n", [(104, 88), (512, 1000)])
@pytest.mark.parametrize("packed", [False, True])
def test_gateup_with_biases(dtype, k, n, packed):
    g = torch.Generator().manual_seed(n)
    both = (_rand(g, n, 2, k) * k ** -0.5).to(dtype)
    bg, bu = _rand(g, n).to(dtype), _rand(g, n).to(dtype)
    dev = both.to(DEV)
    gate, up = (dev[:, 0], dev[:, 1]) if packed else (dev[:, 0].contiguous(), dev[:, 1].contiguous())
    for tokens in (1, 2, 3, 7, 16, 17, 39, 70, 300, 1100):
        x = _rand(g, tokens, k).to(dtype)
        a = x.double() @ both[:, 0].double().T + bg.double()
        ref = a * torch.sigmoid(a) * (x.double() @ both[:, 1].double().T + bu.double())
        _close(muillm_ext.mui_gateup_silu(None, 0.0, gate, up, x.to(DEV), bg.to(DEV), bu.to(DEV)), ref, REL[dtype], tokens)
    with pytest.raises(RuntimeError):
        muillm_ext.mui_gateup_silu(None, 0.0, gate, up, x.to(DEV), bg.to(DEV), None)


def test_gateup_with_biases_over_bands_of_the_prompt_gemm():
    """A size whose outputs are dealt out to two launches: the second one has biases of its own rows."""
    k, n, tokens = 256, 14336, 2048
    g = torch.Generator(device=DEV).manual_seed(3)
    gate, up, x = (torch.randn(*s, device=DEV, generator=g).to(torch.bfloat16) for s in ((n, k), (n, k), (tokens, k)))
    gate, up = gate * k ** -0.5, up * k ** -0.5
    bg, bu = (3 * torch.randn(n, device=DEV, generator=g).to(torch.bfloat16) for _ in range(2))
    y = muillm_ext.mui_gateup_silu(None, 0.0, gate, up, x, bg, bu).float()
    a, b = x.float() @ gate.float().T + bg.float(), x.float() @ up.float().T + bu.float()
    ref = torch.nn.functional.silu(a) * b
    assert float((y - ref).abs().max() / ref.abs().max()) < 1e-2


# --------------------------------------------------------------------------------------
# bigram embedding
# --------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,buckets,mul_prev,mul_cur", [(104, 59, 31, 5), (37, 7, 1, 1), (2056, 997, 1000003, 7)])
def test_bigram_embedding(dtype, width, buckets, mul_prev, mul_cur):
    g = torch.Generator().manual_seed(width)
    vocab, batch, n = 70, 3, 23
    table, bigram = _rand(g, vocab, width).to(dtype), _rand(g, buckets + 1, width).to(dtype)
    ids = torch.randint(0, vocab, (batch, n), generator=g)
    pads = torch.tensor([0, 4, 1])
    prev = torch.full((batch,), 33, device=DEV)
    got_x, got_h, at = [], [], 0
    for cut in (6, 1, 2, 1, 1, 12):
        x, h = ops.bigram_embedding(ids[:, at:at + cut].to(DEV), prev, _slots(at, cut), pads.to(DEV), table.to(DEV), bigram.to(DEV),
                                    2.5, mul_prev, mul_cur)
        at += cut
        got_x.append(x)
        got_h.append(h)
    x, h = torch.cat(got_x, 1), torch.cat(got_h, 1)
    for b in range(batch):
        ref = oracle.embed(ids[b, pads[b]:], table, 2.5, bigram, buckets, mul_prev, mul_cur)
        _close(x[b, pads[b]:], ref, 1e-6, b)
        _close(h[b, pads[b]:], ref, max(REL[dtype] / 3, 1e-6), b)
    assert torch.equal(prev.cpu(), ids[:, -1])


# --------------------------------------------------------------------------------------
# attention
# --------------------------------------------------------------------------------------
PREPARE = [(6, 2, 40, 24, 16), (1, 1, 64, 64, 64), (8, 8, 20, 12, 6), (5, 1, 128, 128, 0), (3, 3, 7, 9, 4), (16, 4, 256, 200, 128)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,rot", PREPARE)
@pytest.mark.parametrize("start,t", [(0, 19), (37, 1), (1000, 3)])
def test_prepare(dtype, heads, kv_heads, dim, vdim, rot, start, t):
    g = torch.Generator().manual_seed(dim + t)
    nq, nk, nv, batch = heads * dim, kv_heads * dim, kv_heads * vdim, 2
    proj = _rand(g, batch, t, nq + nk + nv + 16, std=2.0).to(dtype)
    qg, kg = (1 + 0.3 * _rand(g, nq)).to(dtype), (1 + 0.3 * _rand(g, nk)).to(dtype)
    freq = oracle.frequencies(rot, 50.0, {"factor": 3.0, "high": 4.0, "low": 1.0, "original": 60}) if rot else torch.zeros(0, dtype=torch.float64)
    pads = torch.tensor([0, 2 if start else 0])
    kc = torch.zeros(batch, start + t + 3, nk, dtype=dtype, device=DEV)
    vc = torch.zeros(batch, start + t + 3, nv, dtype=dtype, device=DEV)
    for gains in ((qg, kg), (None, None)):
        dq, dk = (None if x is None else x.to(DEV) for x in gains)
        q = ops.hybrid_prepare(proj.to(DEV), heads, kv_heads, dim, vdim, dq, dk, 0.2, freq.to(DEV), _slots(start, t), pads.to(DEV), kc, vc)
        for b in range(batch):
            pos = torch.arange(start, start + t) - pads[b]
            x, y = proj[b, :, :nq].double(), proj[b, :, nq:nq + nk].double()
            if gains[0] is not None:
                x, y = oracle.rms(x, 0.2) * qg.double(), oracle.rms(y, 0.2) * kg.double()
            ref_q = oracle.rotate_pairs(x.reshape(t, heads, dim), pos, freq).reshape(t, nq)
            ref_k = oracle.rotate_pairs(y.reshape(t, kv_heads, dim), pos, freq).reshape(t, nk)
            _close(q[b], ref_q, max(REL[dtype] / 3, 2e-6), "q")
            _close(kc[b, start:start + t], ref_k, max(REL[dtype] / 3, 2e-6), "k")
            assert torch.equal(vc[b, start:start + t].cpu(), proj[b, :, nq + nk:nq + nk + nv])
        assert start == 0 or float(kc[:, :start].abs().max()) == 0


def test_prepare_far_positions():
    """A million positions on, angles are still those of the exact product."""
    freq = oracle.frequencies(64, 10000.0)
    proj = torch.ones(1, 1, 192)
    kc, vc = torch.zeros(1, 4, 64, device=DEV), torch.zeros(1, 4, 64, device=DEV)
    start = torch.tensor([2 - 1_000_003])
    q = ops.hybrid_prepare(proj.to(DEV), 1, 1, 64, 64, None, None, 0.0, freq.to(DEV), torch.tensor([2], device=DEV), start.to(DEV), kc, vc)
    ref = oracle.rotate_pairs(proj[0, :, :64].reshape(1, 1, 64), torch.tensor([1_000_003]), freq)
    _close(q[0], ref.reshape(1, 64), 1e-6)


def _attend(dtype, q, k, v, gate, scale, softcap, window, keep, past, pads=None, route=None, spare=5):
    """q [B, T, H, d], k / v [B, past + T, G, .]."""
    b, t, heads, dim = q.shape
    kv_heads, vdim, n = k.shape[2], v.shape[3], k.shape[1]
    kc = torch.full((b, n + spare, kv_heads * dim), 7.0, dtype=dtype, device=DEV)  # rows behind the tokens are never read
    vc = torch.full((b, n + spare, kv_heads * vdim), float("nan"), dtype=dtype, device=DEV)
    kc[:, :n] = k.reshape(b, n, -1).to(DEV)
    vc[:, :n] = v.reshape(b, n, -1).to(DEV)
    full = None
    if gate is not None:  # a slice of a wider projection
        full = torch.zeros(b, t, heads * vdim + 8, dtype=dtype, device=DEV)
        full[..., 8:] = gate.to(DEV)
        full = full[..., 8:]
    return ops.hybrid_attention(q.reshape(b, t, -1).to(DEV), kc, vc, full, _slots(past, t), None if pads is None else pads.to(DEV),
                                heads, kv_heads, scale, softcap, window, keep, route)


ATTEND = [  # heads, kv_heads, dim, vdim, window, keep_first, softcap, scale
    (6, 2, 40, 24, 37, 3, 7.5, 0.2), (4, 4, 64, 64, 16, 0, 0.0, 0.12), (8, 2, 96, 128, 130, 70, 20.0, 0.1), (5, 1, 128, 72, 0, 0, 3.0, 0.09),
    (18, 1, 32, 40, 65, 1, 11.0, 0.2), (2, 1, 200, 256, 64, 64, 0.0, 0.07), (4, 2, 20, 12, 9, 2, 5.0, 0.25), (3, 3, 8, 8, 1, 0, 2.0, 0.4),
    (2, 2, 16, 264, 2, 1, 4.0, 0.3), (12, 3, 72, 8, 300, 6, 30.0, 0.1)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", range(len(ATTEND)))
@pytest.mark.parametrize("past,t", [(0, 1), (0, 150), (63, 1), (210, 16), (130, 2), (300, 1), (97, 70), (5, 33)])
def test_attention(dtype, case, past, t):
    heads, kv_heads, dim, vdim, window, keep, softcap, scale = ATTEND[case]
    g = torch.Generator().manual_seed(case * 1000 + past + t)
    n = past + t
    q, k = _rand(g, 1, t, heads, dim, std=1.5).to(dtype), _rand(g, 1, n, kv_heads, dim, std=1.5).to(dtype)
    v, gate = _rand(g, 1, n, kv_heads, vdim).to(dtype), _rand(g, 1, t, heads * vdim).to(dtype)
    ref = oracle.attention(q[0], k[0], v[0], scale, softcap, window, keep, past).reshape(t, -1)
    rel = {torch.float32: 1e-5, torch.bfloat16: 2e-2, torch.float16: 3e-3}[dtype]
    _close(_attend(dtype, q, k, v, gate, scale, softcap, window, keep, past)[0], ref * torch.sigmoid(gate[0].double()), rel, "gated")
    _close(_attend(dtype, q, k, v, None, scale, softcap, window, keep, past)[0], ref, rel, "plain")
    if t > 1:  # a prompt's tokens through the kernels of decoding
        if ops.hybrid_route(dtype, 1, dim, vdim) == _lib.MUI_HYBRID_DECODE:
            _close(_attend(dtype, q, k, v, gate, scale, softcap, window, keep, past, route=_lib.MUI_HYBRID_DECODE)[0],
                   ref * torch.sigmoid(gate[0].double()), rel, "decode route")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("t", [1, 16, 40, 130])
def test_attention_at_every_edge(dtype, t):
    """One key stands out for every query: the oldest one inside the window, the first one outside it, the last kept token or the
    first one that is not; a limit that is one token off in either direction gives a different answer."""
    heads, kv_heads, dim, vdim, window, keep, past = 2, 1, 32, 16, 70, 5, 100
    n = past + t
    g = torch.Generator().manual_seed(t)
    for spot in ("oldest", "outside", "kept", "dropped"):
        key = {"oldest": past + t - window, "outside": past + t - window - 1, "kept": keep - 1, "dropped": keep}[spot]
        q = torch.ones(1, t, heads, dim).to(dtype)
        k = (0.05 * _rand(g, 1, n, kv_heads, dim)).to(dtype)
        k[0, key] = 1.0
        v = _rand(g, 1, n, kv_heads, vdim).to(dtype)
        v[0, key] += 3.0
        got = _attend(dtype, q, k, v, None, 0.4, 30.0, window, keep, past)[0]
        ref = oracle.attention(q[0], k[0], v[0], 0.4, 30.0, window, keep, past).reshape(t, -1)
        rel = {torch.float32: 1e-5, torch.bfloat16: 2e-2, torch.float16: 3e-3}[dtype]
        _close(got, ref, rel, spot)
        off = {"oldest": (window - 1, keep), "outside": (window + 1, keep), "kept": (window, keep - 1), "dropped": (window, keep + 1)}[spot]
        wrong = oracle.attention(q[0], k[0], v[0], 0.4, 30.0, *off, past).reshape(t, -1)
        assert float((got.cpu().double() - wrong).abs().max()) > 0.5, spot


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("past,t", [(0, 90), (90, 1), (83, 7), (60, 30)])
def test_attention_of_padded_batches(dtype, past, t):
    heads, kv_heads, dim, vdim, window, keep = 4, 2, 48, 32, 33, 4
    g = torch.Generator().manual_seed(past)
    n, pads = past + t, torch.tensor([0, 50, 13])
    q, k, v = (_rand(g, 3, m, h, d).to(dtype) for m, h, d in ((t, heads, dim), (n, kv_heads, dim), (n, kv_heads, vdim)))
    got = _attend(dtype, q, k, v, None, 0.2, 9.0, window, keep, past, pads)
    for b in range(3):
        skip = max(0, int(pads[b]) - past)  # tokens of this call that are padding
        ref = oracle.attention(q[b, skip:], k[b, pads[b]:], v[b, pads[b]:], 0.2, 9.0, window, keep, past + skip - int(pads[b]))
        _close(got[b, skip:], ref.reshape(t - skip, -1), {torch.float32: 1e-5, torch.bfloat16: 2e-2, torch.float16: 3e-3}[dtype], b)
        assert skip == 0 or float(got[b, :skip].abs().max()) == 0


# --------------------------------------------------------------------------------------
# gated delta rule
# --------------------------------------------------------------------------------------
class _Delta:
    def __init__(self, dtype, heads, kv_heads, dk, dv, taps, ra=8, rg=16, seed=0, strong=0.0, eps=1e-3):
        g = torch.Generator().manual_seed(seed)
        self.dtype, self.heads, self.kv_heads, self.dk, self.dv = dtype, heads, kv_heads, dk, dv
        nq, nv = kv_heads * dk, heads * dv
        self.widths = {"q": nq, "k": nq, "v": nv, "a": ra, "g": rg, "b": heads}
        self.offsets, at = [], 0
        for w in self.widths.values():
            self.offsets.append(at)
            at += (w + 7) // 8 * 8
        self.pitch, self.eps = at, eps
        self.conv = _rand(g, 2 * nq + nv, taps).to(dtype)
        self.a2, self.g2 = (_rand(g, heads * dk, ra) * 1.5 * ra ** -0.5).to(dtype), (_rand(g, nv, rg) * rg ** -0.5).to(dtype)
        self.dt_bias, self.a_log = (-1.5 + 1.5 * _rand(g, heads * dk)).to(dtype), (0.5 * _rand(g, heads) + strong).to(dtype)
        self.gain = (1 + 0.2 * _rand(g, dv)).to(dtype)
        self.gen = g

    def inputs(self, batch, t):
        return _rand(self.gen, batch, t, self.pitch).to(self.dtype)

    def layer(self):
        c = [x.to(DEV) for x in (self.conv, self.a2, self.dt_bias, self.a_log, self.g2, self.gain)]
        return ops.ChannelDelta(self.heads, self.kv_heads, self.dk, self.dv, tuple(self.offsets), *c, self.eps)

    def states(self, batch):
        layer = self.layer()
        ring = torch.full((batch, layer.ring_rows, layer.channels), float("nan"), dtype=self.dtype, device=DEV)  # rows are written before they are read
        return torch.zeros(batch, self.heads, self.dk, self.dv, device=DEV), ring

    def run(self, proj, cuts, pads=None, states=None):
        layer, (s, ring) = self.layer(), states or self.states(proj.shape[0])
        outs, at = [], 0
        for n in cuts:
            outs.append(ops.channel_delta(layer, proj[:, at:at + n].contiguous().to(DEV), s, ring, _slots(at, n),
                                          None if pads is None else pads.to(DEV)))
            at += n
        assert at == proj.shape[1]
        return torch.cat(outs, 1), s

    def reference(self, proj):
        """One sequence [T, pitch]: (y, S)."""
        t = proj.shape[0]
        part = {n: proj[:, o:o + w].double() for (n, w), o in zip(self.widths.items(), self.offsets)}
        nq = self.kv_heads * self.dk
        q, k, v = (oracle.short_conv(part[n], self.conv[lo:hi]) for n, lo, hi in (("q", 0, nq), ("k", nq, 2 * nq), ("v", 2 * nq, None)))
        q = oracle.unit(q.reshape(t, self.kv_heads, self.dk)) * self.dk ** -0.5
        k = oracle.unit(k.reshape(t, self.kv_heads, self.dk))
        eye = torch.eye(self.a2.shape[1], dtype=torch.float64)
        decay = torch.exp(oracle.log_decay(part["a"], eye, self.a2, self.dt_bias, self.a_log))
        o, s = oracle.channel_delta(q, k, v.reshape(t, self.heads, self.dv), torch.sigmoid(part["b"]), decay)
        gate = torch.sigmoid(part["g"] @ self.g2.double().T)
        return (oracle.rms(o, self.eps) * self.gain.double()).reshape(t, -1) * gate, s


# y is normed per head, which magnifies what is small; S is compared on its own
Y_REL = {torch.float32: 1e-4, torch.bfloat16: 1e-2, torch.float16: 2e-3}

# (heads, kv_heads, dk, dv, taps[, ranks])
DELTA = [(4, 2, 40, 56, 3), (2, 2, 64, 64, 4), (3, 1, 24, 20, 1), (2, 1, 130, 33, 2), (1, 1, 256, 40, 4), (2, 2, 12, 13, 5), (2, 1, 64, 300, 8),
         (1, 1, 264, 16, 4), (2, 1, 16, 16, 9), (2, 2, 128, 128, 4), (1, 1, 200, 72, 6),
         # ranks (of the decay and of the gate) that fill the registers of the step kernel, exceed them, are no multiple of 8
         (2, 2, 128, 128, 4, 128, 128), (1, 1, 128, 256, 4, 64, 24), (2, 1, 48, 72, 4, 200, 13), (2, 1, 100, 40, 2, 72, 136)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", range(len(DELTA)))
def test_delta_rule(dtype, case):
    d = _Delta(dtype, *DELTA[case], seed=case)
    n = 150
    proj = d.inputs(1, n)
    ref, s_ref = d.reference(proj[0])
    for cuts in ([n], [1] * n, [16] * 9 + [6], [17, 2, 64, 3, 1, 1, 62], [63, 65, 22], [2] * 75):
        y, s = d.run(proj, cuts)
        _close(y[0], ref, Y_REL[dtype], cuts[:6])
        _close(s[0], s_ref, 2e-5, cuts[:6])


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("strong", [-8.0, 3.0, 6.0])
def test_delta_rule_with_decays_from_none_to_total(dtype, strong):
    d = _Delta(dtype, 2, 1, 72, 40, 4, seed=11, strong=strong)
    proj = d.inputs(1, 200)
    ref, s_ref = d.reference(proj[0])
    for cuts in ([200], [40, 33, 127], [100] + [1] * 100):
        y, s = d.run(proj, cuts)
        _close(y[0], ref, Y_REL[dtype], cuts[:4])
        _close(s[0], s_ref, 2e-5, cuts[:4])


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_delta_rule_of_padded_batches_and_segments(dtype, monkeypatch):
    d = _Delta(dtype, 4, 2, 32, 24, 4, seed=5)
    n, pads = 140, torch.tensor([0, 77, 3])
    proj = d.inputs(3, n)
    for segment in (4096, 32):  # long prompts go segment by segment
        monkeypatch.setattr(ops, "DELTA_SEGMENT", segment)
        for cuts in ([n], [5, 80, 55], [100] + [1] * 40):
            y, s = d.run(proj, cuts, pads)
            for b in range(3):
                ref, s_ref = d.reference(proj[b, pads[b]:])
                _close(y[b, pads[b]:], ref, Y_REL[dtype], (b, cuts[:3]))
                _close(s[b], s_ref, 2e-5, (b, cuts[:3]))


def test_delta_rule_remembers_one_write():
    """A value written once is read back much later, scaled by the product of the decays in between, across chunk borders."""
    d = _Delta(torch.float32, 1, 1, 16, 16, 1, seed=3)
    n = 300
    for where in (0, 15, 16, 63, 64, 100):
        proj = torch.zeros(1, n, d.pitch)
        proj[..., d.offsets[5]] = -30.0                # beta 0: nothing is written ...
        proj[0, where, d.offsets[5]] = 30.0            # ... but here
        proj[..., d.offsets[0]:d.offsets[0] + 16] = 1.0
        proj[..., d.offsets[1]:d.offsets[1] + 16] = 1.0
        proj[0, where, d.offsets[2]:d.offsets[2] + 16] = torch.arange(16.0)
        d.a_log.fill_(-6.0)
        ref, s_ref = d.reference(proj[0])
        for cuts in ([n], [n - 40] + [1] * 40, [where + 1, n - where - 1]):
            y, s = d.run(proj, cuts)
            _close(y[0, where:], ref[where:], 1e-4, (where, cuts[:2]))
            _close(s[0], s_ref, 1e-5, (where, cuts[:2]))
        assert float(ref[-1].abs().max()) > 0.1
