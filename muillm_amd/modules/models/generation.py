"""MuiGenerationMixin: generate() / generate_greedy() of a causal LM over the device-resident decode loop
(the reference routes generate() through its MuiGenerationMixin._sample,
muillm/sampling/generation.py:77-408)."""
from typing import Optional

import torch

from ..kvcache.cache_utils import MuiCache


class MuiGenerationMixin:
    """Needs of the class: forward() as MuiGraphDecoder calls it, create_cache(), max_positions(),
    pads_in_cache, and a `_graph_decoder` attribute that starts as None."""

    @torch.no_grad()
    def generate_greedy(self, input_ids: torch.LongTensor, max_new_tokens: int, use_graph: Optional[bool] = None,
                        cache: Optional[MuiCache] = None, return_logits: bool = False):
        """Prefill on the prompt, then max_new_tokens greedy decode steps at the prompt's batch
        size. Returns int64 [B, prompt + max_new_tokens] (and, optionally, the per-step fp16
        logits of the decode steps).

        use_graph=True captures the decode step (model forward, argmax, position bookkeeping,
        all on the device) into a HIP graph and replays it; False enqueues the same step on the
        stream every time; None (default) lets the decoder choose (MuiGraphDecoder: stream launches
        when the layer stack is one library call, graph replay otherwise)."""
        dec = self._decoder_for(use_graph=use_graph)
        cache = self._reusable_cache(dec, cache, input_ids)
        return dec.generate(input_ids, max_new_tokens, cache=cache, return_logits=return_logits)

    def _decoder_for(self, **options):
        """The MuiGraphDecoder for these options; the last one is kept, so that repeated generate()
        calls replay the graph captured by the first instead of warming up and capturing again."""
        from .graphdecoder import MuiGraphDecoder

        key = tuple(sorted((k, tuple(v) if isinstance(v, (list, tuple)) else v) for k, v in options.items()))
        if self._graph_decoder is None or self._graph_decoder[0] != key:
            self._graph_decoder = (key, MuiGraphDecoder(self, **options))
        return self._graph_decoder[1]

    @staticmethod
    def _reusable_cache(dec, cache, input_ids):
        """Without a cache from the caller, a kept decoder starts again on its own (emptied) cache
        when the batch size fits: same buffers, so its captured graph stays valid. A cache that a
        caller handed to an earlier call is the caller's (multi-turn state) and is never touched."""
        if cache is None and dec.cache is not None and dec.owns_cache \
                and dec.cache.max_batch_size == input_ids.shape[0] \
                and dec.cache.tensors()[0].device == input_ids.device:
            dec.cache.reset()
            return dec.cache
        return cache

    @torch.no_grad()
    def generate(self, input_ids: torch.LongTensor = None, attention_mask: Optional[torch.Tensor] = None,
                 max_new_tokens: int = 20, do_sample: bool = False, temperature: float = 1.0,
                 top_k: Optional[int] = None, top_p: Optional[float] = None,
                 eos_token_id=None, pad_token_id: Optional[int] = None, seed: int = 0, use_graph: Optional[bool] = None,
                 cache: Optional[MuiCache] = None, **unused):
        """HuggingFace-style entry point over the device-resident decode loop (the reference routes
        generate() through its MuiGenerationMixin._sample, muillm/sampling/generation.py:77-408).
        Greedy (do_sample=False) or temperature sampling; left-padded batches via attention_mask;
        rows stop at eos_token_id (int or list) and are filled with pad_token_id afterwards.
        Returns int64 [B, prompt_len + max_new_tokens]. top_k / top_p filter the logits with torch
        ops in front of the sampling kernel (the loop then runs eagerly instead of from the HIP
        graph); other logit processors (penalties, ...) are not part of this loop."""
        dropped = {k: v for k, v in unused.items() if v is not None and k in ("repetition_penalty", "num_beams")}
        if dropped:
            raise NotImplementedError(f"generate(): unsupported options {sorted(dropped)}")
        eos = None
        if eos_token_id is not None:
            eos = [int(eos_token_id)] if isinstance(eos_token_id, int) else [int(e) for e in eos_token_id]
        if pad_token_id is None:
            pad_token_id = eos[0] if eos else 0
        dec = self._decoder_for(use_graph=use_graph, eos_token_ids=eos, pad_token_id=pad_token_id,
                                do_sample=do_sample, temperature=temperature, seed=seed,
                                top_k=top_k if do_sample else None, top_p=top_p if do_sample else None)
        cache = self._reusable_cache(dec, cache, input_ids)
        # with an eos criterion the loop polls, without blocking, whether every row has finished
        return dec.generate(input_ids, max_new_tokens, cache=cache, attention_mask=attention_mask,
                            stop_check_every=8 if eos else 0)
