"""What every language model of the library shares on the Python side: the calls over the generation runtime that each
model exports under its own prefix (agpu_gpt2_*, agpu_ritevik_*, agpu_piralix_*)."""
import ctypes as C

import numpy as np

from . import _lib
from ._lib import AgpuError


def _np(a, dtype):
    return np.ascontiguousarray(a, dtype=dtype)


class LanguageModel:
    """A device-resident model with a cache.  A subclass sets `prefix`, `default_eos` (-1: none), `config` (with vocab_size and
    max_batch), `ctx`, `_lib` and `handle`."""

    prefix = None
    default_eos = -1
    DECODE_AUTO, DECODE_PER_STAGE, DECODE_EAGER = 0, 1, 2

    def _check(self, rc):
        if rc != 0:
            raise AgpuError(rc, self._lib.agpu_last_error_string(self.ctx.handle).decode())

    def _eos(self, eos):
        return self.default_eos if eos is None else eos

    def _call(self, name, *args):
        fn = getattr(self._lib, name)
        conv = [_lib.ptr(a) if (t is C.c_void_p) else a for a, t in zip(args, fn.argtypes[1:])]
        self._check(fn(self.handle, *conv))

    def close(self):
        if getattr(self, "handle", None):
            getattr(self._lib, self.prefix + "_destroy")(self.handle)
            self.handle = None

    def __del__(self):
        try:
            self.close()
        except Exception:
            pass

    def reset_cache(self):
        self._call(self.prefix + "_reset_cache")

    def cache_len(self):
        return int(getattr(self._lib, self.prefix + "_cache_len")(self.handle))

    def forward_cached(self, tokens, all_rows=True):
        """tokens [batch, new_len] (numpy); returns logits as numpy, [batch, new_len, V] or [batch, V]."""
        tokens = np.atleast_2d(_np(tokens, np.uint32))
        B, n = tokens.shape
        V = self.config.vocab_size
        p = C.c_void_p()
        self.ctx.call("agpu_malloc", tokens.nbytes, C.byref(p))
        rows = B * n if all_rows else B
        lg = C.c_void_p()
        self.ctx.call("agpu_malloc", rows * V * 4, C.byref(lg))
        try:
            self.ctx.call("agpu_memcpy_h2d", p.value, tokens, tokens.nbytes)
            self._call(self.prefix + "_forward_cached", p.value, B, n, lg.value, int(all_rows))
            out = np.empty((B, n, V) if all_rows else (B, V), np.float32)
            self.ctx.call("agpu_memcpy_d2h", out, lg.value, out.nbytes)
        finally:
            self.ctx.call("agpu_free", p.value)
            self.ctx.call("agpu_free", lg.value)
        return out

    def forward(self, tokens):
        """Int4Gpt2Model::forward (gpt2.rs:1522-1533): uncached, logits [seq, V] of one sequence."""
        self.reset_cache()
        return self.forward_cached(np.asarray(tokens).reshape(1, -1), all_rows=True)[0]

    def generate_cached(self, prompt, max_new_tokens, eos=None):
        """Returns (list of token arrays per sequence, (prefill_ms, decode_ms))."""
        prompt = np.atleast_2d(_np(prompt, np.uint32))
        B, n = prompt.shape
        out = np.zeros((B, n + max_new_tokens), np.uint32)
        lens = np.zeros(B, np.int32)
        ms = np.zeros(2, np.float32)
        self._call(self.prefix + "_generate_cached", prompt, B, n, max_new_tokens, self._eos(eos), out, lens, ms)
        return [out[b, :lens[b]].copy() for b in range(B)], (float(ms[0]), float(ms[1]))

    def generate_text(self, tokenizer, prompt, max_new_tokens, eos=None):
        """Text in, text out, as the reference's callers do around the model (tokenizer.encode(prompt) -> tokens ->
        generate -> tokenizer.decode, gpt2.rs:1619-1630, 1790-1836): greedy continuation of `prompt`, prompt included."""
        tokens = tokenizer.encode(prompt)
        if not tokens:
            raise ValueError("empty prompt")
        (out,), _ = self.generate_cached(np.asarray(tokens, np.uint32), max_new_tokens, eos=eos)
        return tokenizer.decode(out.tolist())

    def generate_cached_sampling(self, prompt, max_new_tokens, top_k, temperature, rng, eos=None):
        """Int4Gpt2Model::generate_cached_sampling (gpt2.rs:931-977); rng is an ops.SimpleRng and is advanced."""
        prompt = _np(prompt, np.uint32).ravel()
        out = np.zeros(prompt.size + max_new_tokens, np.uint32)
        n = C.c_int32(0)
        self._call(self.prefix + "_generate_cached_sampling", prompt, prompt.size, max_new_tokens, top_k, float(temperature),
                   C.addressof(rng._s), self._eos(eos), out, C.addressof(n))
        return out[: n.value].copy()

    def generate(self, prompt, max_new_tokens, eos=None):
        prompt = _np(prompt, np.uint32).ravel()
        out = np.zeros(prompt.size + max_new_tokens, np.uint32)
        n = C.c_int32(0)
        self._call(self.prefix + "_generate", prompt, prompt.size, max_new_tokens, self._eos(eos), out, C.addressof(n))
        return out[: n.value].copy()

    def decode_steps(self, batch, steps):
        """Replays `steps` decode steps from the current state; returns the total milliseconds."""
        ms = C.c_float(0)
        self._call(self.prefix + "_decode_steps", batch, steps, C.addressof(ms))
        return float(ms.value)

    def set_decode_mode(self, mode):
        """DECODE_AUTO: single-sequence steps run as one launch where the shape allows; DECODE_PER_STAGE: one launch per stage,
        replayed as a HIP graph; DECODE_EAGER: the same launches without a graph."""
        self._call(self.prefix + "_set_decode_mode", mode)

    def last_logits(self, batch=1):
        """[batch, vocab] logits of the last position as the most recent forward or decode step left them."""
        out = np.empty((batch, self.config.vocab_size), np.float32)
        self._call(self.prefix + "_last_logits", batch, out)
        return out
