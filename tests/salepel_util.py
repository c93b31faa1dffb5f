"""Small Salepel configurations and random weights for the tests."""
import torch


def latent(heads=3, dim=24, rot=8, vdim=40, q_rank=56, kv_rank=48, window=37, scale=None, base=5000.0, kv_from=None, **_):
    mx = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
          "mask": {"size": window}, "rot": {"base": base, "dims": rot},
          "scale": (dim + rot) ** -0.5 if scale is None else scale}
    if kv_from is not None:
        mx["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": mx}


def mlstm(heads=2, dim=40, vdim=72, cap=9.0):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def moe(experts=5, identity=2, top=3, ff=56, limit=0.7):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit},
            "router": {"experts": experts, "identity": identity, "top": top}}


def config(layers, width=96, vocab=136, eps=3e-5, embed_scale=5.5):
    """layers: (mixer entry, feed-forward or None) pairs."""
    return {"architecture": "Salepel", "embedding": {"scale": embed_scale}, "norm": {"eps": eps}, "vocab": vocab, "width": width,
            "layers": [dict(m, mlp=f) for m, f in layers]}


def default_config(window=37, **kw):
    return config([(mlstm(), moe()), (latent(window=window), moe(identity=0, top=2)), (latent(window=window - 16, kv_from=1), None),
                   (mlstm(heads=3, dim=24, vdim=20), None), (latent(heads=5, window=window + 20), moe(experts=3, identity=4, top=4))], **kw)


def random_weights(cfg, seed=0, dtype=torch.bfloat16, sharp=2.0, close_calls=True):
    """{tensor name: tensor}: matrices ~ N(0, 1 / in), gains around 1, gate biases that make memories last;
    `sharp` scales the query maps so that attention singles keys out. Values are exact in bf16.
    close_calls=False: for runs in 16 bits. The routers' corrections lie further apart than the scores
    move, so that rounding does not change which experts a token takes, and attention is softer."""
    sharp = sharp if close_calls else 0.5 * sharp
    g = torch.Generator().manual_seed(seed)
    w = {}

    def mat(name, out, inp, gain=1.0):
        w[name] = torch.randn(out, inp, generator=g) * gain * inp ** -0.5

    def vec(name, n, mean=1.0, std=0.2):
        w[name] = mean + std * torch.randn(n, generator=g)

    width = cfg["width"]
    mat("embed", cfg["vocab"], width, width ** 0.5 / cfg["embedding"]["scale"])
    for i, layer in enumerate(cfg["layers"]):
        p, mx, ff = f"l{i}.", layer["mixer"], layer["mlp"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if ff else ()):
            vec(p + n, width)
        p += "mix."
        if layer["type"] == "latent_attention":
            h = mx["heads"]
            mat(p + "dq", mx["q_rank"], width)
            vec(p + "dq.norm", mx["q_rank"])
            mat(p + "uq", h * (mx["dim"] + mx["rot_dim"]), mx["q_rank"], sharp)
            if "kv_from" not in mx:
                mat(p + "dkv", mx["kv_rank"] + mx["rot_dim"], width)
                vec(p + "dkv.norm", mx["kv_rank"])
            mat(p + "uk", h * mx["dim"], mx["kv_rank"])
            mat(p + "uv", h * mx["vdim"], mx["kv_rank"])
            mat(p + "o", width, h * mx["vdim"])
        else:
            h, qk, v = mx["heads"], mx["heads"] * mx["dim"], mx["heads"] * mx["vdim"]
            for n, rows in (("q", qk), ("k", qk), ("v", v), ("g", v)):
                mat(p + n, rows, width)
            vec(p + "norm", v)
            mat(p + "i", h, width, 2.0)
            mat(p + "f", h, width, 2.0)
            vec(p + "i.b", h, 0.0)
            vec(p + "f.b", h, 3.0, 1.0)
            mat(p + "o", width, v)
        if ff:
            p = f"l{i}.mlp."
            n = ff["router"]["experts"] + ff["router"].get("identity", 0)
            mat(p + "router", n, width, 1.5 if close_calls else 0.25)
            vec(p + "correction", n, 0.0, 0.05)
            if not close_calls:
                w[p + "correction"] = torch.randperm(n, generator=g) * (2.0 / n)
            for e in range(ff["router"]["experts"]):
                mat(f"{p}e{e}.gate", ff["expert"]["ff"], width)
                mat(f"{p}e{e}.up", ff["expert"]["ff"], width)
                mat(f"{p}e{e}.down", width, ff["expert"]["ff"])
    vec("final.norm", width)
    mat("head", cfg["vocab"], width)
    return {k: t.to(torch.bfloat16).to(dtype) for k, t in w.items()}


def build(cfg, weights, dtype, device="cuda"):
    from muillm_amd.modules.models.salepel.config import MuiSalepelConfig
    from muillm_amd.modules.models.salepel.model import MuiSalepelForCausalLM

    return MuiSalepelForCausalLM.from_tensors(MuiSalepelConfig.from_dict(cfg), weights, dtype=dtype, device=device)


def row_error(got, ref):
    """Per row: rms of the difference over the rms of all of ref."""
    got, ref = got.detach().to("cpu", torch.float64), ref.to(torch.float64)
    assert got.shape == ref.shape and bool(torch.isfinite(got).all())
    return (got - ref).pow(2).mean(-1).sqrt() / ref.pow(2).mean().sqrt()


# rms error of a row of logits against the float64 oracle, relative to the logits' scale
TOL = {torch.float32: 1e-4, torch.bfloat16: 0.08}


def assert_rows(err, dtype, what=""):
    """fp32: every row within TOL. 16 bits: rows at which a memory's n . q (or its whole output) happens to be
    near zero magnify the rounding of their inputs, so a few may lie outside, half of them far inside."""
    worst = f"{what}: row {int(err.argmax())} {float(err.max()):.2e}, median {float(err.median()):.2e}"
    over = float((err > TOL[dtype]).double().mean())
    if dtype == torch.float32:
        assert over == 0, worst
    else:
        assert over <= 0.04 and float(err.median()) < 0.25 * TOL[dtype] and float(err.max()) < 1.0, worst
