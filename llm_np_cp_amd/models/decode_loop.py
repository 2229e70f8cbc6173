"""Generation loops every GPU engine shares.

An engine supplies the forward pass and the one-token step:

    reset(), forward(ids, cache, pos0), forward_full(ids, ...)
    _decode_step(greedy, min_p, temperature)
    _decode_batch_step(B, greedy, min_p, temperature)
    prefill_batch(prompts), prefill_row(b, ids, ...), compact_row(dst, src)

and the device-side decode state (sampled token, RNG counter, output ring,
sequence lengths).  The loops here prefill, sample the first token from
the prefill logits, capture the step in a hipGraph and replay it; the host
sees token ids only once per chunk.  ``_reserve(lens)`` runs before any
step that lets row b grow to lens[b] tokens, for engines whose cache is
allocated on demand.
"""

from __future__ import annotations

from typing import List, Optional

import numpy as np
import torch

from ..ops import hip_ops as ho
from ..parallel import tp as tpu
from ..utils.tracing import trace_range


class DeviceCacheHandle:
    """Host-side mirror of the device seq-length (generate()-compatible)."""

    def __init__(self, engine):
        self.engine = engine
        self.seq_len = 0


class DecodeLoop:
    def _reserve(self, lens: List[int]) -> None:
        """Cache room for row b up to lens[b] tokens (preallocated pools
        have it already)."""

    def make_cache(self, n: int) -> DeviceCacheHandle:
        if n > self.max_seq:
            raise ValueError(f"requested cache {n} > max_seq {self.max_seq}")
        self.reset()
        return DeviceCacheHandle(self)

    def forward_hf(self, ids: np.ndarray):
        """Reference-parity output tuple ``(loss, logits, kv_cache,
        hidden_states, attentions)`` (llama3.2_model.py:726-822).
        ``loss`` is None (inference-only, as in the reference) and
        ``attentions`` is None by design: the fused attention kernels
        use online softmax and never materialize the probability
        matrix."""
        logits, hidden = self.forward_full(ids, return_hidden_states=True)
        cache = DeviceCacheHandle(self)
        cache.seq_len = len(np.ravel(ids))
        return None, logits, cache, hidden, None

    def generate_tokens(self, prompt_ids, max_tokens: int,
                        greedy: bool = True, min_p: float = 0.1,
                        eos_id=None, chunk: int = 16, on_ids=None,
                        temperature: float = 1.0, stop_fn=None):
        """Fast generate: device-side hipGraph decode in chunks, host
        sees ids every `chunk` tokens (streaming + EOS stop).  Used by
        runtime.generate() for greedy/min-p on GPU models.
        ``eos_id`` may be an int or a collection of ints (HF configs
        often store a list, e.g. Llama-3.2-Instruct).  ``stop_fn``
        (optional) sees the accumulated ids after each chunk and returns
        True to end generation early (stop-string support; the caller
        truncates — chunking may have produced up to chunk-1 extra
        ids)."""
        import time as _time
        prompt_ids = np.asarray(prompt_ids)
        room = self.max_seq - len(prompt_ids.ravel()) - 1
        if room <= 0:
            raise ValueError(f"prompt fills the {self.max_seq}-token pool")
        max_tokens = min(max_tokens, room)
        eos_set = (set() if eos_id is None else
                   {int(eos_id)} if np.isscalar(eos_id) else
                   {int(e) for e in eos_id})
        t0 = _time.perf_counter()
        with trace_range("prefill"):
            self.prefill(prompt_ids)
        self.last_prefill_time_s = _time.perf_counter() - t0
        out = []
        produced = 0
        first = True
        with trace_range("decode"):
            while produced < max_tokens:
                n = min(chunk, max_tokens - produced)
                ids = self.decode(n, greedy=greedy, min_p=min_p,
                                  use_graph=True, first_from_logits=first,
                                  temperature=temperature)
                first = False
                produced += n
                stop = False
                take = list(ids)
                hit = [j for j, t in enumerate(take) if int(t) in eos_set]
                if hit:
                    take = take[:hit[0] + 1]
                    stop = True
                out.extend(take)
                if on_ids:
                    on_ids(take)
                if stop:
                    break
                if stop_fn is not None and stop_fn(out):
                    break
        return out

    def decode_batch(self, n_tokens: int, greedy: bool = True,
                     min_p: float = 0.1, temperature: float = 1.0,
                     use_graph: bool = True,
                     first_from_logits: bool = True) -> np.ndarray:
        """Decode n_tokens for every prefilled sequence; returns int32
        ids of shape (B, n_tokens).  ``first_from_logits=False``
        continues a previous decode_batch (chunked serving)."""
        B = self._batch_n
        if max(self._host_lens) + n_tokens > self.max_seq:
            raise ValueError("decode_batch would overflow the KV pool")
        self._host_lens = [p + n_tokens for p in self._host_lens]
        self._reserve(self._host_lens[:B])
        if first_from_logits:
            # first tokens from the prefill logits (fp32, batch rows)
            ho.sample(self.bt_logits32[:B], min_p, greedy, self.seed,
                      self.rng_ctr, self.bt_gmax, self.bt_pick,
                      self.bt_next, self.bt_ring, self.bt_nout,
                      self.bt_lens, bump_len=False,
                      temperature=temperature, cnt=self.bt_cnt, batch=B)
        n_steps = n_tokens - (1 if first_from_logits else 0)
        key = ("batch", B, greedy, min_p, temperature)
        if use_graph and n_steps > 0 and self._graph_mode != key \
                and not getattr(self, "_graph_failed", False):
            s = torch.cuda.Stream()
            s.wait_stream(torch.cuda.current_stream())
            with torch.cuda.stream(s):
                self._decode_batch_step(B, greedy, min_p, temperature)
            torch.cuda.current_stream().wait_stream(s)
            torch.cuda.synchronize()
            n_steps -= 1
            try:
                g = torch.cuda.CUDAGraph()
                with torch.cuda.graph(g):
                    self._decode_batch_step(B, greedy, min_p, temperature)
                self._graph = g
                self._graph_mode = key
            except Exception as e:
                self._graph_failed = True
                self._graph_error = e
                use_graph = False
        if use_graph and self._graph_mode == key:
            for _ in range(n_steps):
                self._graph.replay()
        else:
            for _ in range(n_steps):
                self._decode_batch_step(B, greedy, min_p, temperature)
        torch.cuda.synchronize()
        n = int(self.bt_nout[0].item())
        out = self.bt_ring[:B, :n].cpu().numpy()
        return out[:, max(0, n - n_tokens):]

    def decode_rows(self, B: int, n: int, greedy: bool = True,
                    min_p: float = 0.1, temperature: float = 1.0,
                    use_graph: bool = True):
        """n lockstep steps for rows [0, B) (each already holding a
        sampled next token from prefill_row / a previous chunk).
        Returns a list of B arrays: each row's n new token ids."""
        assert 1 <= B <= self.max_batch
        if max(self._host_lens[:B]) + n > self.max_seq:
            raise ValueError("decode_rows would overflow the KV pool")
        for b in range(B):
            self._host_lens[b] += n
        self._reserve(self._host_lens[:B])
        key = ("batchc", B, greedy, min_p, temperature)
        if not hasattr(self, "_bgraphs"):
            self._bgraphs = {}
        g = self._bgraphs.get(key)
        executed = 0
        if (use_graph and g is None and n > 1
                and not getattr(self, "_graph_failed", False)):
            s = torch.cuda.Stream()
            s.wait_stream(torch.cuda.current_stream())
            with torch.cuda.stream(s):
                self._decode_batch_step(B, greedy, min_p, temperature)
            torch.cuda.current_stream().wait_stream(s)
            torch.cuda.synchronize()
            executed += 1  # the warm-up was a real step
            try:
                g = torch.cuda.CUDAGraph()
                with torch.cuda.graph(g):
                    self._decode_batch_step(B, greedy, min_p, temperature)
                self._bgraphs[key] = g
            except Exception as e:
                self._graph_failed = True
                self._graph_error = e
                g = None
        remaining = n - executed
        if g is not None and use_graph:
            for _ in range(remaining):
                g.replay()
        else:
            for _ in range(remaining):
                self._decode_batch_step(B, greedy, min_p, temperature)
        torch.cuda.synchronize()
        comm = tpu.xgmi_comm()
        if comm is not None:
            comm.check()
        nouts = self.bt_nout[:B].cpu().numpy()
        ring = self.bt_ring[:B].cpu().numpy()
        # each step appends exactly one id per row
        return [ring[b, max(0, int(nouts[b]) - n):int(nouts[b])]
                for b in range(B)]

    def generate_tokens_batch(self, prompts, max_tokens: int,
                              greedy: bool = True, min_p: float = 0.1,
                              temperature: float = 1.0) -> np.ndarray:
        """Convenience: prefill_batch + decode_batch -> (B, max_tokens)."""
        self.prefill_batch(prompts)
        return self.decode_batch(max_tokens, greedy=greedy, min_p=min_p,
                                 temperature=temperature)

    def capture_decode_graph(self, greedy: bool = True, min_p: float = 0.1,
                             temperature: float = 1.0):
        """Capture one decode step into a hipGraph (fixed shapes: KV pool
        is preallocated and the position is a device scalar, so the graph
        is shape-stable).

        NOTE: the warm-up executes ONE REAL decode step (advances the
        sequence by one token).  Returns ``(steps_taken, ok)``:
        ``steps_taken`` is the number of real decode steps executed here
        (1 whenever the warm-up ran, 0 when the cached graph is reused)
        — callers MUST account for it even when ``ok`` is False.  On
        capture failure ``ok`` is False, ``self._graph_failed`` is set
        (no further capture attempts) and the exception is kept in
        ``self._graph_error``."""
        mode = (greedy, min_p, temperature)
        if self._graph_mode == mode:
            return 0, True
        if getattr(self, "_graph_failed", False):
            return 0, False
        # warm-up (a real step) on a side stream, then capture
        s = torch.cuda.Stream()
        s.wait_stream(torch.cuda.current_stream())
        with torch.cuda.stream(s):
            self._decode_step(greedy, min_p, temperature)
        torch.cuda.current_stream().wait_stream(s)
        torch.cuda.synchronize()
        try:
            g = torch.cuda.CUDAGraph()
            with torch.cuda.graph(g):
                self._decode_step(greedy, min_p, temperature)
        except Exception as e:
            # the warm-up step above DID run (token committed to
            # out_ring, len_buf advanced) — report it so decode() does
            # not double-count
            self._graph_failed = True
            self._graph_error = e
            torch.cuda.synchronize()
            return 1, False
        self._graph = g
        self._graph_mode = mode
        return 1, True

    def prefill(self, ids: np.ndarray, cache: Optional[DeviceCacheHandle] = None):
        cache = cache or self.make_cache(self.max_seq)
        with trace_range(f"prefill[{len(np.asarray(ids).ravel())}]"):
            logits = self.forward(ids, cache, 0)
        return cache, logits

    def decode(self, n_tokens: int, greedy: bool = True, min_p: float = 0.1,
               use_graph: bool = True, first_from_logits: bool = True,
               temperature: float = 1.0):
        """Generate n_tokens ids device-side; returns int32 numpy ids.
        Assumes prefill() ran (len_buf == prompt length, logits ready)."""
        if getattr(self, "_host_len", 0) + n_tokens > self.max_seq:
            raise ValueError(
                f"decode would overflow the KV pool: len {self._host_len} "
                f"+ {n_tokens} > max_seq {self.max_seq}")
        self._host_len += n_tokens
        self._reserve([self._host_len])
        if first_from_logits:
            # sample token 0 from the prefill logits
            ho.sample(self.b_logits, min_p, greedy, self.seed, self.rng_ctr,
                      self.s_gmax, self.s_pick, self.next_token,
                      self.out_ring, self.nout, self.len_buf,
                      bump_len=False, temperature=temperature,
                      cnt=self.s_cnt)
        n_steps = n_tokens - (1 if first_from_logits else 0)
        if use_graph and n_steps > 0:
            # capture_decode_graph reports the warm-up step it executed
            # even when capture fails, so n_steps stays exact either way
            taken, ok = self.capture_decode_graph(greedy, min_p, temperature)
            n_steps -= taken
            if not ok:
                use_graph = False
        if use_graph and n_steps > 0:
            for _ in range(n_steps):
                self._graph.replay()
        else:
            for _ in range(n_steps):
                self._decode_step(greedy, min_p, temperature)
        torch.cuda.synchronize()
        comm = tpu.xgmi_comm()
        if comm is not None:
            comm.check()  # raise if a one-shot collective timed out
        n = int(self.nout.item())
        return self.out_ring[:n].cpu().numpy()[max(0, n - n_tokens):]
