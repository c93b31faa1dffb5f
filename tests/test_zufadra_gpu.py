"""The Zufadra decoder on the GPU against the float64 oracle: whole prompts, decoding, portions, batches, reused caches,
generation through the decode loop, and the trace runner."""
import io
import json

import numpy as np
import pytest
import torch

from oracle import zufadra as oracle
from tests.zufadra_util import TOL, assert_rows, attention, build, config, default_config, delta, dense, random_weights, row_error

pytestmark = pytest.mark.gpu
DEV = "cuda"
DTYPES = [torch.float32, torch.bfloat16]


def _tokens(n, vocab, seed=0):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def _in_portions(lm, tokens, cuts, cache=None):
    """Logits of every position, the prompt cut as `cuts` says (the rest token by token)."""
    cache = lm.create_cache(1, 16) if cache is None else cache
    outs, at = [], 0
    for n in list(cuts) + [1] * (len(tokens) - sum(cuts)):
        ids = torch.tensor([tokens[at:at + n]], device=DEV)
        outs.append(lm(input_ids=ids, past_key_values=cache).logits[0])
        at += n
    assert cache.get_seq_length() == len(tokens)
    return torch.cat(outs)


def _no_bigram(cfg):
    del cfg["embedding"]["bigram"]
    return cfg


CONFIGS = {
    "mixed": default_config(),
    "wide_window": default_config(window=500),
    "window_2": config([(attention(window=2, keep_first=1), None), (attention(heads=1, kv_heads=1, window=1, keep_first=0), dense()),
                        (attention(window=3, keep_first=40, scaling=None), None)]),
    "recurrent": config([(delta(), None), (delta(heads=1, kv_heads=1, dim=100, vdim=36, conv=1), dense()), (delta(heads=6, kv_heads=2, conv=2), None)]),
    "odd_sizes": config([(attention(heads=2, kv_heads=1, dim=20, vdim=12, rot=6, window=11), dense(23)),
                         (delta(heads=3, kv_heads=1, dim=11, vdim=13, conv=4), dense(9))], width=51, vocab=67, bigram=(1, 0, 0)),
    "large_heads": config([(attention(heads=18, kv_heads=1, dim=96, vdim=168, rot=96, window=65, keep_first=64, softcap=50.0), dense(64)),
                           (delta(heads=2, kv_heads=1, dim=160, vdim=136, conv=4), None)], width=192, mult=1.0, logit_scale=1.0, embed_scale=1.0),
    "no_bigram": _no_bigram(default_config()),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", CONFIGS)
def test_prompt_portions_and_decoding(name, dtype):
    cfg = CONFIGS[name]
    w = random_weights(cfg, seed=len(name))
    tokens = _tokens(150, cfg["vocab"])
    ref, _ = oracle.forward(cfg, w, tokens)
    lm = build(cfg, w, dtype)
    # once through the prompt, token by token, and cut in several ways (down to two tokens)
    for cuts in ([150], [], [120], [2] * 75, [40, 2, 30, 17, 16, 3, 2, 35], [1, 2, 64, 65], [16, 17, 100]):
        assert_rows(row_error(_in_portions(lm, tokens, cuts), ref), dtype, f"cuts {cuts[:8]}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_residual_stream_after_every_layer(dtype):
    cfg = default_config()
    w = random_weights(cfg, seed=3)
    tokens = _tokens(60, cfg["vocab"], 3)
    _, ref = oracle.forward(cfg, w, tokens)
    out = build(cfg, w, dtype)(input_ids=torch.tensor([tokens], device=DEV), output_hidden_states=True)
    for i, x in enumerate(out.hidden_states):
        assert x.dtype == torch.float32
        assert_rows(row_error(x[0], ref[i]), dtype, f"layer {i}")


def test_limits_that_are_one_token_off_would_be_seen():
    """The weights of these tests tell a window or a number of kept tokens that is one off from rounding."""
    cfg = default_config()
    w = random_weights(cfg, seed=5)
    tokens = _tokens(150, cfg["vocab"])
    ref, _ = oracle.forward(cfg, w, tokens)
    lm = build(cfg, w, torch.float32)
    got = _in_portions(lm, tokens, [100])
    assert float(row_error(got, ref).max()) < TOL[torch.float32]
    for plant in ({"window": -1}, {"window": 1}, {"keep_first": -1}, {"keep_first": 1}):
        wrong, _ = oracle.forward(cfg, w, tokens, plant=plant)
        assert float(row_error(got, wrong).max()) > 50 * TOL[torch.float32], plant


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(dtype):
    cfg = default_config(window=48)
    w = random_weights(cfg, seed=7)
    tokens = _tokens(400, cfg["vocab"], 7)
    ref, _ = oracle.forward(cfg, w, tokens)
    assert_rows(row_error(_in_portions(build(cfg, w, dtype), tokens, [9]), ref), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_reused_and_grown_caches(dtype):
    cfg = default_config()
    w = random_weights(cfg, seed=8)
    lm = build(cfg, w, dtype)
    cache = lm.create_cache(1, 8)
    for seed, n, cuts in ((1, 140, [90]), (2, 33, [2, 2]), (3, 170, [170]), (4, 1, [1]), (5, 77, [70, 2])):
        tokens = _tokens(n, cfg["vocab"], seed)
        cache.reset()
        if dtype != torch.float32 and n < 20:  # too few rows for shares of them
            _in_portions(lm, tokens, cuts, cache)
            continue
        assert_rows(row_error(_in_portions(lm, tokens, cuts, cache), oracle.forward(cfg, w, tokens)[0]), dtype, seed)
    assert cache.max_cache_len == 256


@pytest.mark.parametrize("dtype", DTYPES)
def test_batch_rows_equal_single_rows(dtype):
    cfg = default_config()
    w = random_weights(cfg, seed=9)
    lm = build(cfg, w, dtype)
    rows = [_tokens(90, cfg["vocab"], s) for s in (1, 2, 3)]
    cache = lm.create_cache(3, 90)
    ids = torch.tensor(rows, device=DEV)
    got = torch.cat([lm(input_ids=ids[:, a:b], past_key_values=cache).logits for a, b in ((0, 70), (70, 72), (72, 90))], 1)
    for i, tokens in enumerate(rows):
        assert_rows(row_error(got[i], oracle.forward(cfg, w, tokens)[0]), dtype, i)


@pytest.mark.parametrize("dtype", DTYPES)
def test_left_padded_batch_equals_single_rows(dtype):
    cfg = default_config()
    w = random_weights(cfg, seed=10)
    lm = build(cfg, w, dtype)
    rows = [_tokens(n, cfg["vocab"], n) for n in (60, 43, 25)]
    ids = torch.tensor([[0] * (60 - len(r)) + r for r in rows], device=DEV)
    mask = torch.tensor([[0] * (60 - len(r)) + [1] * len(r) for r in rows], device=DEV)
    cache = lm.create_cache(3, 64)
    more = torch.tensor([_tokens(6, cfg["vocab"], 50 + i) for i in range(3)], device=DEV)
    got = [lm(input_ids=ids, attention_mask=mask, past_key_values=cache).logits]
    got += [lm(input_ids=more[:, i:i + 1], past_key_values=cache).logits for i in range(6)]
    got = torch.cat(got, 1)
    for i, r in enumerate(rows):
        ref, _ = oracle.forward(cfg, w, r + more[i].tolist())
        assert_rows(row_error(got[i, 60 - len(r):], ref), dtype, i)


def _check_greedy(cfg, w, prompt, tokens, tol):
    """Every generated token is (up to rounding) the oracle's best continuation of what precedes it."""
    seq = tokens.tolist()
    logits, _ = oracle.forward(cfg, w, seq[:-1])
    scale = float(logits.pow(2).mean().sqrt())
    for p in range(len(prompt) - 1, len(seq) - 1):
        assert float(logits[p].max() - logits[p, seq[p + 1]]) <= tol * scale, p


def test_greedy_generation_through_the_decode_loop():
    cfg = default_config()
    w = random_weights(cfg, seed=11)
    lm = build(cfg, w, torch.bfloat16)
    prompt = _tokens(21, cfg["vocab"], 1)
    ids = torch.tensor([prompt], device=DEV)
    eager = lm.generate_greedy(ids, 70, use_graph=False)
    _check_greedy(cfg, w, prompt, eager[0].cpu(), 4 * TOL[torch.bfloat16])
    # captured steps, replayed in several calls with other work between them: the same tokens every time
    for use_graph in (True, None, True):
        torch.randn(1000, device=DEV).sum().item()
        assert torch.equal(lm.generate_greedy(ids, 70, use_graph=use_graph), eager)
    other = torch.tensor([_tokens(35, cfg["vocab"], 2)], device=DEV)
    assert torch.equal(lm.generate_greedy(other, 40, use_graph=True), lm.generate_greedy(other, 40, use_graph=False))


def test_generate_batch_with_padding_and_eos():
    cfg = default_config()
    w = random_weights(cfg, seed=12)
    lm = build(cfg, w, torch.bfloat16)
    rows = [_tokens(30, cfg["vocab"], 1), _tokens(11, cfg["vocab"], 2)]
    ids = torch.tensor([[0] * (30 - len(r)) + r for r in rows], device=DEV)
    mask = torch.tensor([[0] * (30 - len(r)) + [1] * len(r) for r in rows], device=DEV)
    for use_graph in (True, False):
        out = lm.generate(ids, attention_mask=mask, max_new_tokens=24, use_graph=use_graph)
        for i, r in enumerate(rows):
            _check_greedy(cfg, w, r, out[i, 30 - len(r):].cpu(), 4 * TOL[torch.bfloat16])
    single = lm.generate(torch.tensor([rows[0]], device=DEV), max_new_tokens=24)
    eos = int(single[0, 30 + 5])
    stopped = lm.generate(torch.tensor([rows[0]], device=DEV), max_new_tokens=24, eos_token_id=eos, pad_token_id=7)[0, 30:].tolist()
    first = single[0, 30:].tolist().index(eos)
    assert stopped[:first + 1] == single[0, 30:].tolist()[:first + 1] and set(stopped[first + 1:]) <= {7}
    sampled = [lm.generate(ids, attention_mask=mask, max_new_tokens=8, do_sample=True, seed=3) for _ in range(2)]
    assert torch.equal(*sampled)


def test_trace_replay(tmp_path):
    from safetensors.torch import save_file

    from muillm_amd import trace
    from muillm_amd.modules.models.registry import load_model

    cfg = default_config()
    w = random_weights(cfg, seed=13)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    lm = load_model(str(tmp_path), dtype=torch.float32, device=DEV)
    a, b = _tokens(80, cfg["vocab"], 1), _tokens(30, cfg["vocab"], 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:50], "want": [0, 49]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[50:79], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[79:], "want": [0]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": b[:2], "want": [1, 0]}], "end": []},
             {"step": 4, "entries": [{"id": "b", "tokens": b[2:], "want": [27]}], "end": ["b"]}]
    said = []
    trace.run(lm, DEV, io.StringIO("".join(json.dumps(s) + "\n" for s in steps)), str(tmp_path), 64, said.append)
    assert said == [f"done {i}" for i in range(5)] and not (tmp_path / "1.f32").exists()
    ra, rb = oracle.forward(cfg, w, a)[0], oracle.forward(cfg, w, b)[0]
    for step, ref in ((0, ra[[0, 49]]), (2, ra[[79]]), (3, rb[[1, 0]]), (4, rb[[29]])):
        got = torch.from_numpy(np.fromfile(tmp_path / f"{step}.f32", dtype="<f4").copy()).reshape(-1, cfg["vocab"])
        assert float(row_error(got, ref).max()) < TOL[torch.float32], step
