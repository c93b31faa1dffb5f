"""Small Zufadra configurations and random weights for the tests."""
import torch

from tests.salepel_util import row_error  # noqa: F401


def attention(heads=6, kv_heads=2, dim=40, vdim=24, window=37, keep_first=3, rot=16, base=5000.0, scaling=(3.0, 2.5, 1.5, 90),
              scale=None, softcap=7.5):
    """scaling: (factor, high, low, original)."""
    rot = {"base": base, "dims": rot}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "high", "low", "original"), scaling))
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                                           "mask": {"size": window, "keep_first": keep_first}, "rot": rot,
                                           "scale": dim ** -0.5 if scale is None else scale, "softcap": softcap}}


def delta(heads=4, kv_heads=2, dim=40, vdim=56, conv=3):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def dense(ff=88):
    return {"kind": "dense", "ff": ff}


def config(layers, width=104, vocab=136, eps=3e-5, embed_scale=2.5, mult=0.7, logit_scale=0.3, bigram=(59, 5, 31)):
    """layers: (mixer entry, feed-forward or None) pairs; bigram: (buckets, mul_cur, mul_prev)."""
    return {"architecture": "Zufadra", "embedding": {"scale": embed_scale, "bigram": dict(zip(("buckets", "mul_cur", "mul_prev"), bigram))},
            "norm": {"eps": eps}, "residual_mult": mult, "logit_scale": logit_scale, "vocab": vocab, "width": width,
            "layers": [dict(m, mlp=f) for m, f in layers]}


def default_config(window=37, **kw):
    return config([(delta(), dense()), (attention(window=window), None), (attention(window=window + 20, keep_first=1), dense(64)),
                   (delta(heads=3, kv_heads=3, dim=24, vdim=24, conv=4), None)], **kw)


def random_weights(cfg, seed=0, dtype=torch.bfloat16, sharp=2.0, ranks=(12, 20)):
    """{tensor name: tensor}: matrices ~ N(0, 1 / in), gains around 1; decays from nearly none to strong; `sharp` scales
    the queries so that attention singles keys out. ranks: of the decay and of the gate. Values are exact in bf16."""
    g = torch.Generator().manual_seed(seed)
    w = {}

    def mat(name, out, inp, gain=1.0):
        w[name] = torch.randn(out, inp, generator=g) * gain * inp ** -0.5

    def vec(name, n, mean=1.0, std=0.2):
        w[name] = mean + std * torch.randn(n, generator=g)

    width, e = cfg["width"], cfg["embedding"]
    mat("embed", cfg["vocab"], width, width ** 0.5 / e["scale"])
    if "bigram" in e:
        mat("bigram", e["bigram"]["buckets"] + 1, width, 0.7 * width ** 0.5)
    for i, layer in enumerate(cfg["layers"]):
        p, mx, ff = f"l{i}.", layer["mixer"], layer["mlp"]
        vec(p + "norm1", width)
        h, kvh, dim, vdim = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
        p += "mix."
        mat(p + "k", kvh * dim, width)
        if layer["type"] == "attention":
            mat(p + "q", h * dim, width)
            mat(p + "v", kvh * vdim, width)
            mat(p + "g", h * vdim, width)
            vec(p + "q.norm", h * dim, sharp, 0.3 * sharp)
            vec(p + "k.norm", kvh * dim)
        else:
            mat(p + "q", kvh * dim, width)
            mat(p + "v", h * vdim, width)
            for n, c in (("q", kvh * dim), ("k", kvh * dim), ("v", h * vdim)):
                mat(f"{p}{n}.conv", c, mx["conv"], 1.3)
            mat(p + "b", h, width)
            mat(p + "a1", ranks[0], width)
            mat(p + "a2", h * dim, ranks[0], 2.0)
            vec(p + "dt_bias", h * dim, -2.5, 2.0)
            vec(p + "A_log", h, 0.0, 0.7)
            mat(p + "g1", ranks[1], width)
            mat(p + "g2", h * vdim, ranks[1])
            vec(p + "norm", vdim)
        mat(p + "o", width, h * vdim)
        if ff:
            vec(f"l{i}.norm2", width)
            p = f"l{i}.mlp."
            for n, out, inp in (("gate", ff["ff"], width), ("up", ff["ff"], width), ("down", width, ff["ff"])):
                mat(p + n, out, inp)
                vec(p + n + ".b", out, 0.0, 0.5)
    vec("final.norm", width)
    mat("head", cfg["vocab"], width)
    return {k: t.to(torch.bfloat16).to(dtype) for k, t in w.items()}


def build(cfg, weights, dtype, device="cuda"):
    from muillm_amd.modules.models.zufadra.config import MuiZufadraConfig
    from muillm_amd.modules.models.zufadra.model import MuiZufadraForCausalLM

    return MuiZufadraForCausalLM.from_tensors(MuiZufadraConfig.from_dict(cfg), weights, dtype=dtype, device=device)


# rms error of a row of logits against the float64 oracle, relative to the logits' scale
TOL = {torch.float32: 1e-4, torch.bfloat16: 0.08}


def assert_rows(err, dtype, what=""):
    """fp32: every row within TOL. 16 bits: rows at which a head's output happens to be near zero before its norm magnify
    the rounding of their inputs, so a few may lie outside, half of them far inside."""
    worst = f"{what}: row {int(err.argmax())} {float(err.max()):.2e}, median {float(err.median()):.2e}"
    over = float((err > TOL[dtype]).double().mean())
    if dtype == torch.float32:
        assert over == 0, worst
    else:
        assert over <= 0.05 and float(err.median()) < 0.4 * TOL[dtype] and float(err.max()) < 1.0, worst
