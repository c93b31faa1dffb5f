"""Host logic of the Zufadra decoder: configuration, tensor names, cache bookkeeping, registry; and the oracle of its
mechanisms against closed forms."""
import copy
import json
import math

import pytest
import torch

from muillm_amd import _lib
from muillm_amd.engineconfig import MuiEngineConfig
from muillm_amd.modules.attention.rotaryembedding import compute_rope_inv_freq
from muillm_amd.modules.kvcache.hybridcache import MuiHybridCache
from muillm_amd.modules.models.registry import architecture_of
from muillm_amd.modules.models.zufadra.config import MuiZufadraConfig
from muillm_amd.modules.models.zufadra.model import MuiZufadraForCausalLM
from oracle import zufadra as oracle
from tests.zufadra_util import attention, config, default_config, delta, dense, random_weights


def _lm(cfg, w, dtype=torch.float32):
    return MuiZufadraForCausalLM.from_tensors(MuiZufadraConfig.from_dict(cfg), w, dtype=dtype, device="cpu",
                                              engine_config=MuiEngineConfig())


def test_config_reads_every_size_and_refuses_what_cannot_be():
    cfg = default_config()
    c = MuiZufadraConfig.from_dict(cfg)
    assert (c.hidden_size, c.vocab_size, c.num_hidden_layers, c.residual_mult, c.logit_scale) == (104, 136, 4, 0.7, 0.3)
    a, d = c.layers[1].mixer, c.layers[0].mixer
    assert (a.window, a.keep_first, a.softcap, a.rot_dims, c.layers[2].mixer.window) == (37, 3, 7.5, 16, 57)
    assert (d.taps, d.heads, d.kv_heads) == (3, 4, 2) and c.layers[1].ff is None and c.layers[2].ff == 64
    assert (c.bigram.buckets, c.bigram.mul_cur, c.bigram.mul_prev) == (59, 5, 31)
    no_mlp_key = copy.deepcopy(cfg)
    del no_mlp_key["layers"][1]["mlp"]
    assert MuiZufadraConfig.from_dict(no_mlp_key) == c

    def broken(change):
        bad = copy.deepcopy(cfg)
        change(bad)
        with pytest.raises((ValueError, KeyError)):
            MuiZufadraConfig.from_dict(bad)

    broken(lambda d: d.update(architecture="other"))
    broken(lambda d: d.pop("residual_mult"))
    broken(lambda d: d["layers"][0].update(type="other"))
    broken(lambda d: d["layers"][0]["mixer"].pop("conv"))
    broken(lambda d: d["layers"][0]["mixer"].update(conv=0))
    broken(lambda d: d["layers"][0]["mixer"].update(kv_heads=3))
    broken(lambda d: d["layers"][1]["mixer"].update(kv_heads=4))
    broken(lambda d: d["layers"][1]["mixer"]["mask"].update(size=0))
    broken(lambda d: d["layers"][1]["mixer"]["rot"].update(dims=5))
    broken(lambda d: d["layers"][1]["mixer"]["rot"]["scaling"].pop("low"))
    broken(lambda d: d["layers"][0]["mlp"].update(kind="moe"))
    broken(lambda d: d["embedding"]["bigram"].update(buckets=0))
    with pytest.warns(UserWarning, match="extra"):
        MuiZufadraConfig.from_dict(dict(cfg, extra=1))


def test_every_tensor_finds_its_place():
    cfg = default_config()
    w = random_weights(cfg, seed=1, ranks=(11, 17))
    lm = _lm(cfg, w, torch.bfloat16)
    names = dict(lm.checkpoint_tensors())
    assert set(names) == set(w)
    for n, t in names.items():
        assert torch.equal(t, w[n]), n
    assert "l1.norm2" not in names and "l0.norm2" in names
    # whatever is not covered is the zero padding of the low-rank parts
    covered = sum(t.numel() for t in names.values())
    assert sum(p.numel() for p in lm.parameters()) - covered == sum(
        (16 - 11 + 24 - 17 + 8 - h) * 104 + h * (5 * d + 7 * v) for h, d, v in ((4, 40, 56), (3, 24, 24)))
    mixer = lm.model.layers[0].mixer
    assert float(mixer.decay_up[:, 11:].abs().max()) == 0 and float(mixer.proj.linear.weight[-4:].abs().max()) == 0
    for bad in ({k: v for k, v in w.items() if k != "l0.mix.k.conv"}, dict(w, extra=torch.zeros(1)), dict(w, head=torch.zeros(3, 3)),
                {k: v for k, v in w.items() if k != "l3.mix.a1"}):
        with pytest.raises(ValueError):
            _lm(cfg, bad)


def test_cache_holds_rows_memories_and_the_last_token():
    cfg = default_config()
    lm = _lm(cfg, random_weights(cfg))
    cache = lm.create_cache(2, 50)
    assert isinstance(cache, MuiHybridCache) and cache.max_cache_len == 64
    assert cache.layers[1].k.shape == (2, 64, 80) and cache.layers[1].v.shape == (2, 64, 48)
    memory, ring = cache.layers[0].values
    assert memory.shape == (2, 4, 40, 56) and memory.dtype == torch.float32
    assert ring.shape == (2, 2 + _lib.MUI_MAX_TOKENS, 2 * 80 + 224)
    assert cache.front.values[0].shape == (2,) and cache.front.values[0].dtype == torch.int64
    assert len(cache.step_state()) == 5 and len(cache.tensors()) == 5 + 4
    cache.layers[1].k.normal_()
    memory.normal_()
    kept = cache.layers[1].k.clone()
    cache.grow_cache(65)
    assert cache.max_cache_len == 128 and torch.equal(cache.layers[1].k[:, :64], kept)
    cache.set_seen_tokens(65)
    cache.reset()
    assert cache.get_seq_length() == 0 and float(memory.abs().max()) == 0
    assert not lm.takes_embeddings
    with pytest.raises(ValueError):
        lm.model(inputs_embeds=torch.zeros(1, 2, 104), past_key_values=cache)


def test_without_bigram_embedding_rows_are_enough():
    cfg = default_config()
    del cfg["embedding"]["bigram"]
    w = random_weights(cfg)
    lm = _lm(cfg, w)
    assert lm.takes_embeddings and lm.create_cache(1, 8).front is None and "bigram" not in dict(lm.checkpoint_tensors())


def test_registry_goes_by_config_json(tmp_path):
    (tmp_path / "config.json").write_text(json.dumps(default_config()))
    assert architecture_of(str(tmp_path)) == "Zufadra"


def test_frequencies_of_the_module_equal_the_oracles():
    for dims, base, (factor, high, low, original) in ((16, 5000.0, (3.0, 2.5, 1.5, 90)), (24, 100.0, (8.0, 4.0, 1.0, 4096)), (2, 10.0, (2.0, 3.0, 1.0, 5))):
        scaling = {"factor": factor, "low_freq_factor": low, "high_freq_factor": high, "original_max_position_embeddings": original}
        got, _ = compute_rope_inv_freq("llama3", base, dims, scaling, dtype=torch.float64)
        ref = oracle.frequencies(dims, base, {"factor": factor, "high": high, "low": low, "original": original})
        assert got.dtype == torch.float64 and torch.allclose(got, ref, rtol=1e-13, atol=0)


def test_argument_checks_need_no_gpu():
    lib = _lib.load()
    assert lib.mui_bigram_embedding(None, 1, None, None, None, None, None, None, 1.0, 1, 1, 5, None, None, 1, 1, 8, 8) == -1
    assert lib.mui_hybrid_prepare(None, 1, None, 8, 0, 0, None, None, 0.0, None, 0, None, None, None, None, 0, None, 0, 1, 1, 1, 1, 8, 8, 8) == -1
    assert lib.mui_channel_delta(None, 1, None, None, 8, None, None, None, None, None, None, 1, 1) == -1
    assert lib.mui_gateup_silu_bias(None, 1, None, None, 8, None, None, 0.0, None, None, None, 8, 8, 1) == -1
    assert lib.mui_hybrid_attention_route(2, 100, 64, 64) == _lib.MUI_HYBRID_PLAIN
    assert lib.mui_hybrid_attention_route(1, 100, 64, 60) == _lib.MUI_HYBRID_PLAIN
    assert lib.mui_hybrid_attention_route(1, 100, 264, 64) == _lib.MUI_HYBRID_PLAIN
    assert lib.mui_hybrid_attention_route(1, 16, 64, 72) == _lib.MUI_HYBRID_DECODE
    assert lib.mui_hybrid_attention_route(0, 17, 256, 8) == _lib.MUI_HYBRID_PREFILL
    assert lib.mui_channel_delta_ring_rows(4) == 19 and lib.mui_channel_delta_workspace_bytes(1, 16, 2, 8, 8) == 0
    assert lib.mui_channel_delta_workspace_bytes(1, 17, 2, 8, 8) > 0
    assert lib.mui_channel_delta_max_tokens(264, 4) == lib.mui_channel_delta_max_tokens(64, 9) == 16
    assert lib.mui_channel_delta_max_tokens(256, 8) > 1 << 20


# ---- the oracle itself ----------------------------------------------------------------------
def test_oracle_rotation_is_relative_and_partial():
    f = oracle.frequencies(8, 100.0)
    x, y = torch.randn(1, 1, 12, dtype=torch.float64), torch.randn(1, 1, 12, dtype=torch.float64)
    a = oracle.rotate_pairs(x.expand(5, 1, 12), torch.arange(5), f)
    b = oracle.rotate_pairs(y.expand(5, 1, 12), torch.arange(5), f)
    assert torch.equal(a[..., 8:], x.expand(5, 1, 12)[..., 8:]) and torch.allclose(a[:1], x)
    assert torch.allclose((a[1] * b[0]).sum(), (a[4] * b[3]).sum())
    # the first pair turns by one radian a position
    assert torch.allclose(a[1, 0, 0], x[0, 0, 0] * math.cos(1) - x[0, 0, 1] * math.sin(1))


def test_oracle_bigram_rows():
    rows = oracle.bigram_rows(torch.tensor([3, 7, 7, 0]), 10, 4, 9)
    assert rows.tolist() == [10, (12 + 63) % 10, (28 + 63) % 10, 28 % 10]


def test_oracle_visibility_with_sinks():
    seen = oracle.visible(torch.arange(8), torch.arange(8), 3, 2)
    assert seen[7].tolist() == [True, True, False, False, False, True, True, True]
    assert seen[3].tolist() == [True, True, True, True] + [False] * 4
    assert oracle.visible(torch.arange(4), torch.arange(4), None, 0).sum() == 10


def test_oracle_delta_rule_closed_forms():
    """With orthonormal keys and beta 1 the memory returns what was written; writing a key again replaces its value;
    decay acts on key channels; a write of half strength goes half the way."""
    e = torch.eye(3, dtype=torch.float64)
    k = e[[0, 1, 0]][:, None]
    v = torch.tensor([[[1.0, 2.0]], [[3.0, 4.0]], [[5.0, 6.0]]], dtype=torch.float64)
    one, keep = torch.ones(3, 1, dtype=torch.float64), torch.ones(3, 1, 3, dtype=torch.float64)
    o, s = oracle.channel_delta(k, k, v, one, keep)
    assert torch.allclose(o, v) and torch.allclose(s[0], torch.tensor([[5.0, 6.0], [3.0, 4.0], [0.0, 0.0]], dtype=torch.float64))
    _, s = oracle.channel_delta(k[:2], k[:2], v[:2], one[:2], keep[:2] * torch.tensor([0.5, 1.0, 1.0], dtype=torch.float64))
    assert torch.allclose(s[0, 0], 0.5 * v[0, 0]) and torch.allclose(s[0, 1], v[1, 0])
    _, s = oracle.channel_delta(k, k, v, 0.5 * one, keep)
    assert torch.allclose(s[0, 0], 0.25 * v[0, 0] + 0.5 * v[2, 0])
    # two value heads over one key head, state carried over a cut
    v2 = torch.cat([v, -v], 1)
    o, s = oracle.channel_delta(k, k, v2, one.repeat(1, 2), keep.repeat(1, 2, 1))
    _, half = oracle.channel_delta(k[:2], k[:2], v2[:2], one[:2].repeat(1, 2), keep[:2].repeat(1, 2, 1))
    o2, s2 = oracle.channel_delta(k[2:], k[2:], v2[2:], one[2:].repeat(1, 2), keep[2:].repeat(1, 2, 1), half)
    assert torch.allclose(o[:, 1], -o[:, 0]) and torch.allclose(o2[0], o[2]) and torch.allclose(s2, s)


def test_oracle_short_convolution():
    x = torch.arange(1.0, 5.0, dtype=torch.float64)[:, None]
    y = oracle.short_conv(x, torch.tensor([[10.0, 1.0]]))
    z = torch.tensor([1.0, 12.0, 23.0, 34.0], dtype=torch.float64)[:, None]
    assert torch.allclose(y, z / (1 + torch.exp(-z)))


def test_oracle_sees_planted_mistakes():
    cfg = config([(attention(window=9, keep_first=2), dense()), (delta(), None)])
    w = random_weights(cfg, seed=2)
    tokens = list(range(40))
    a, _ = oracle.forward(cfg, w, tokens)
    b, _ = oracle.forward(cfg, w, tokens, plant={"window": 1})
    assert torch.allclose(a[:11], b[:11]) and float((a[11:] - b[11:]).abs().max()) > 1e-2
    b, _ = oracle.forward(cfg, w, tokens, plant={"keep_first": 1})
    assert torch.allclose(a[:11], b[:11]) and float((a[11:] - b[11:]).abs().max()) > 1e-2
