"""Host logic of the Salepel decoder: configuration, tensor names, cache bookkeeping, registry, trace runner
options; and the oracle of its mechanisms against closed forms."""
import copy
import json
import math

import pytest
import torch

from muillm_amd.engineconfig import MuiEngineConfig
from muillm_amd.modules.kvcache.hybridcache import MuiCachePool, MuiHybridCache
from muillm_amd.modules.models.registry import architecture_of
from muillm_amd.modules.models.salepel.config import MuiSalepelConfig
from muillm_amd.modules.models.salepel.model import MuiSalepelForCausalLM
from oracle import salepel as oracle
from tests.salepel_util import config, default_config, latent, mlstm, moe, random_weights


def _lm(cfg, w, dtype=torch.float32):
    return MuiSalepelForCausalLM.from_tensors(MuiSalepelConfig.from_dict(cfg), w, dtype=dtype, device="cpu",
                                              engine_config=MuiEngineConfig())


def test_config_reads_every_size_and_refuses_what_cannot_be():
    cfg = default_config()
    c = MuiSalepelConfig.from_dict(cfg)
    assert (c.hidden_size, c.vocab_size, c.num_hidden_layers) == (96, 136, 5)
    assert c.layers[2].mixer.kv_source == 1 and c.layers[2].mixer.window == 21 and c.layers[2].mlp is None
    assert c.layers[1].mlp.identity == 0 and c.layers[3].mixer.gate_cap == 9.0
    no_mlp_key = copy.deepcopy(cfg)
    del no_mlp_key["layers"][2]["mlp"]
    assert MuiSalepelConfig.from_dict(no_mlp_key) == c

    def broken(change):
        bad = copy.deepcopy(cfg)
        change(bad)
        with pytest.raises((ValueError, KeyError)):
            MuiSalepelConfig.from_dict(bad)

    broken(lambda d: d.update(architecture="other"))
    broken(lambda d: d["layers"][0].update(type="other"))
    broken(lambda d: d["layers"][0]["mixer"].pop("gate_cap"))
    broken(lambda d: d["layers"][1]["mixer"]["rot"].update(dims=4))
    broken(lambda d: d["layers"][1]["mixer"]["mask"].update(size=0))
    broken(lambda d: d["layers"][2]["mixer"].update(kv_from=0))   # a recurrent layer
    broken(lambda d: d["layers"][2]["mixer"].update(kv_from=4))   # comes later
    broken(lambda d: d["layers"][4]["mixer"].update(kv_from=2))   # has no rows of its own
    broken(lambda d: d["layers"][2]["mixer"].update(kv_rank=40))
    broken(lambda d: d["layers"][0]["mlp"]["router"].update(top=8))
    broken(lambda d: d["layers"][0]["mlp"].update(kind="dense"))
    with pytest.warns(UserWarning, match="extra"):
        MuiSalepelConfig.from_dict(dict(cfg, extra=1))


def test_every_tensor_finds_its_place():
    cfg = default_config()
    w = random_weights(cfg, seed=1)
    lm = _lm(cfg, w, torch.bfloat16)
    names = dict(lm.checkpoint_tensors())
    assert set(names) == set(w)
    for n, t in names.items():
        assert torch.equal(t, w[n]), n
    assert "l2.mix.dkv" not in names and "l2.norm2" not in names
    # all of every parameter is covered
    assert sum(t.numel() for t in names.values()) == sum(p.numel() for p in lm.parameters())
    for bad in ({k: v for k, v in w.items() if k != "l0.mix.i.b"}, dict(w, extra=torch.zeros(1)), dict(w, head=torch.zeros(3, 3))):
        with pytest.raises(ValueError):
            _lm(cfg, bad)


def test_hybrid_cache_bookkeeping():
    cfg = default_config()
    lm = _lm(cfg, random_weights(cfg))
    cache = lm.create_cache(2, 50)
    assert isinstance(cache, MuiHybridCache) and cache.max_cache_len == 64
    assert cache.layers[2] is None and cache.layers[1].c.shape == (2, 64, 48)
    assert len(cache.step_state()) == 6 and len(cache.tensors()) == 6 + 4
    cache.layers[1].c.normal_()
    cache.layers[0].values[0].normal_()
    kept = cache.layers[1].c.clone()
    cache.grow_cache(65)
    assert cache.max_cache_len == 128 and torch.equal(cache.layers[1].c[:, :64], kept)
    cache.set_seen_tokens(65)
    cache.set_row_start(torch.tensor([0, 3]))
    assert cache.row_start.data_ptr() in [t.data_ptr() for t in cache.tensors()]
    cache.reset()
    assert cache.get_seq_length() == 0 and cache.row_start is None and float(cache.layers[0].values[0].abs().max()) == 0
    with pytest.raises(ValueError):
        lm.model(input_ids=None)


def test_cache_pool_hands_caches_back_clean():
    made = []

    class Cache:
        def __init__(self):
            made.append(self)
            self.resets = 0

        def reset(self):
            self.resets += 1

    pool = MuiCachePool(Cache)
    a, b = pool.get("a"), pool.get("b")
    assert pool.get("a") is a and a is not b and len(made) == 2
    pool.release("a")
    pool.release("unknown")
    c = pool.get("c")
    assert c is a and c.resets == 1 and pool.get("a") is not a


def test_registry_goes_by_config_json(tmp_path):
    (tmp_path / "config.json").write_text(json.dumps(default_config()))
    assert architecture_of(str(tmp_path)) == "Salepel"
    (tmp_path / "config.json").write_text(json.dumps({"architectures": ["LlamaForCausalLM"]}))
    assert architecture_of(str(tmp_path)) == "LlamaForCausalLM"
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "unheard of"}))
    with pytest.raises(ValueError):
        architecture_of(str(tmp_path))


def test_trace_runner_options():
    from muillm_amd import trace

    a = trace._parse(["--model", "m", "--dtype", "float32", "--out", "o", "--max-tokens", "99"])
    assert (a.model, a.dtype, a.out, a.max_tokens) == ("m", "float32", "o", 99)
    with pytest.raises(SystemExit):
        trace._parse(["--model", "m", "--out", "o", "--dtype", "int4"])


def test_argument_checks_need_no_gpu():
    from muillm_amd import _lib

    lib = _lib.load()
    assert lib.mui_residual_norm(None, 1, None, None, 1.0, None, 1.0, None, 1.0, 0.0, None, None, 1, 8) == -1
    assert lib.mui_moe_route(None, 1, None, None, 4, 0, 2, 1, 0, None, None, None, None) == -1
    assert lib.mui_mlstm(None, 1, None, None, None, 8, None, 1.0, 1.0, None, None, None, None, None, None, None, 1, 1, 1, 8, 8) == -1
    assert lib.mui_moe_tile_pairs(2, 100, 2, 4, 64, 64) == 0 and lib.mui_moe_tile_pairs(1, 4, 2, 4, 64, 63) == 0
    assert lib.mui_moe_tile_pairs(1, 4, 2, 4, 64, 64) == 16 and lib.mui_moe_tile_pairs(1, 4000, 2, 4, 64, 64) == 256
    assert lib.mui_moe_tile_pairs(1, 100, 2, 4, 64, 64) == 128 and lib.mui_moe_tile_pairs(1, 20, 2, 4, 64, 64) == 16
    # enough tiles whatever the routing: every expert may leave one tile part empty
    for tokens, top, experts, tile in ((1, 3, 5, 16), (100, 2, 3, 16), (1000, 4, 60, 128)):
        n = lib.mui_moe_max_tiles(tokens, top, experts, tile)
        assert n >= math.ceil(tokens * top / tile) and n >= min(experts, tokens * top)
    assert lib.mui_mlstm_slices(33) == 2 and lib.mui_mlstm_workspace_bytes(1, 16, 2, 8, 8) == 0
    assert lib.mui_latent_attention_route(2, 100, 8, 64, 16, 64, 128) == _lib.MUI_LATENT_PLAIN
    assert lib.mui_latent_attention_route(1, 1, 3, 24, 8, 40, 48) == _lib.MUI_LATENT_DECODE
    assert lib.mui_latent_attention_route(1, 100, 3, 24, 8, 40, 48) == _lib.MUI_LATENT_PREFILL
    assert lib.mui_latent_attention_route(1, 100, 3, 300, 8, 40, 48) == _lib.MUI_LATENT_DECODE
    assert lib.mui_latent_attention_route(1, 1, 3, 24, 8, 40, 640) == _lib.MUI_LATENT_PLAIN
    assert lib.mui_latent_attention_route(1, 1, 3, 24, 8, 40, 52) == _lib.MUI_LATENT_PLAIN


# ---- the oracle itself ----------------------------------------------------------------------
def test_oracle_rotation_is_relative_and_partial():
    x = torch.randn(1, 12, dtype=torch.float64)
    a = oracle.rotate(x.expand(5, 12), torch.arange(5), 8, 100.0)
    assert torch.equal(a[:, 8:], x.expand(5, 12)[:, 8:]) and torch.allclose(a[0], x[0])
    y = torch.randn(1, 12, dtype=torch.float64)
    b = oracle.rotate(y.expand(5, 12), torch.arange(5), 8, 100.0)
    assert torch.allclose((a[1] * b[0]).sum(), (a[4] * b[3]).sum())


def test_oracle_mlstm_closed_forms():
    """One token: the state is k v^T with a weight, the output does not depend on m where n . q is large;
    a forget gate of log 1/2 halves what is remembered."""
    k, v = torch.tensor([[[1.0, 0.0]]]), torch.tensor([[[3.0, -1.0, 2.0]]])
    q = torch.tensor([[[10.0, 5.0]]])
    zero = torch.zeros(1, 1)
    o, (s, n, m) = oracle.mlstm(q, k, v, zero, zero, 15.0)
    assert torch.allclose(o[0, 0], v[0, 0].double(), atol=1e-5) and float(m) == 0.0
    assert torch.allclose(s[0, 0], v[0, 0].double()) and torch.allclose(s[0, 1], torch.zeros(3, dtype=torch.float64))
    o, (s, n, m) = oracle.mlstm(q.repeat(2, 1, 1), torch.cat([k, 0 * k]), v.repeat(2, 1, 1), torch.zeros(2, 1), torch.zeros(2, 1), 15.0)
    assert abs(float(n[0, 0]) - 0.5) < 1e-12 and abs(float(m)) < 1e-12
    # m never falls below what the running forget gate leaves of its start at 0
    _, (_, _, m) = oracle.mlstm(q, k, v, zero - 9.0, zero + 4.0, 15.0)
    f = math.log(1 / (1 + math.exp(-15 * math.tanh(4 / 15))))
    assert abs(float(m) - f) < 1e-12


def test_oracle_router_and_identity_experts():
    h = torch.eye(4, dtype=torch.float64) * 9
    w = torch.eye(4, dtype=torch.float64)
    chosen, weight = oracle.router(h, w, torch.zeros(4), 1)
    assert chosen.flatten().tolist() == [0, 1, 2, 3]
    assert torch.allclose(weight, torch.full((4, 1), math.exp(9) / (math.exp(9) + 3), dtype=torch.float64))
    chosen, weight2 = oracle.router(h, w, torch.tensor([0.0, 0.0, 0.0, 5.0]), 1)  # the correction chooses, but does not weigh
    assert chosen.flatten().tolist() == [3, 3, 3, 3] and float(weight2[0]) < 1e-3
    y = oracle.moe(h, w, torch.zeros(4), [], 4, 1.0)  # identity experts only, all chosen: the weights add up to 1
    assert torch.allclose(y, h)


def test_oracle_sees_planted_window():
    cfg = config([(latent(window=9), moe()), (mlstm(), None)])
    w = random_weights(cfg, seed=2)
    tokens = list(range(40))
    a, _ = oracle.forward(cfg, w, tokens)
    b, _ = oracle.forward(cfg, w, tokens, plant={"window": 1})
    assert torch.allclose(a[:9], b[:9]) and float((a[9:] - b[9:]).abs().max()) > 1e-2
