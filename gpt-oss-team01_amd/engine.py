"""The engine behind the C ABI for hosts that need no PyTorch: open a model, run steps over rows of any
sequences, read logits, generate."""
from __future__ import annotations

import ctypes as C

import numpy as np

from . import lib as _l


def _ptr(a):
    return a.ctypes.data_as(C.c_void_p)


class Engine:
    """One model on one GPU, with `max_batch` cache slots of up to `max_seq` positions."""

    def __init__(self, cfg, weights_flat=None, max_batch=8, max_seq=64, synthetic=False,
                 precise=False, seed=0, keep_logits=True, prefill=True, mxfp4_experts=False):
        """GPT-OSS from a configuration and a flat fp32 payload (or synthetic weights)."""
        self.L = _l.load()
        self.cfg = cfg
        self._cc = _l.Config.from_config(cfg)
        wp = None
        if not synthetic:
            self._w = np.ascontiguousarray(weights_flat, dtype=np.float32)
            wp = _ptr(self._w)
        h = C.c_void_p()
        _l.check(self.L.gptoss_engine_create(C.byref(self._cc), wp, max_batch, max_seq,
                                             self._flags(synthetic, precise, keep_logits, prefill, mxfp4_experts),
                                             C.c_uint64(seed), C.byref(h)))
        self._adopt(h)

    @classmethod
    def open(cls, path, max_batch=8, max_seq=0, synthetic=False, precise=False, seed=0, keep_logits=True,
             prefill=True, mxfp4_experts=False):
        """Any registered model: a folder with config.json and model.safetensors, or a flat .bin file."""
        e = cls.__new__(cls)
        e.L = _l.load()
        e.cfg = None
        h = C.c_void_p()
        _l.check(e.L.gptoss_engine_open(str(path).encode(), max_batch, max_seq,
                                        cls._flags(synthetic, precise, keep_logits, prefill, mxfp4_experts),
                                        C.c_uint64(seed), C.byref(h)))
        e._adopt(h)
        return e

    @staticmethod
    def _flags(synthetic, precise, keep_logits, prefill, mxfp4_experts):
        return (_l.ENGINE_SYNTHETIC if synthetic else 0) | (_l.ENGINE_PRECISE if precise else 0) | \
            (_l.ENGINE_LOGITS if keep_logits else 0) | (0 if prefill else _l.ENGINE_NO_PREFILL) | \
            (_l.ENGINE_MXFP4_EXPERTS if mxfp4_experts else 0)

    def _adopt(self, handle):
        self._h = handle
        self.info = _l.ModelInfo()
        _l.check(self.L.gptoss_engine_info(handle, C.byref(self.info)))
        self.max_batch, self.max_seq = self.info.max_batch, self.info.max_seq

    def step(self, tokens, pos):
        tok = np.ascontiguousarray(tokens, dtype=np.int32)
        nxt = np.empty_like(tok)
        _l.check(self.L.gptoss_engine_step(self._h, _ptr(tok), int(pos),
                                           tok.size, _ptr(nxt)))
        return nxt

    def prefill(self, tokens):
        """Positions 0..T-1 of every sequence (tokens int32 [B, T]) in one pass -> next ids [B]."""
        tok = np.ascontiguousarray(tokens, dtype=np.int32)
        B, T = tok.shape
        nxt = np.empty(B, np.int32)
        _l.check(self.L.gptoss_engine_prefill(self._h, _ptr(tok), B, T,
                                              _ptr(nxt)))
        return nxt

    def step_ragged(self, tokens, positions):
        """One step with every sequence at its own position."""
        tok = np.ascontiguousarray(tokens, dtype=np.int32)
        pos = np.ascontiguousarray(positions, dtype=np.int32)
        nxt = np.empty_like(tok)
        _l.check(self.L.gptoss_engine_step_ragged(self._h, _ptr(tok),
                                                  _ptr(pos), tok.size,
                                                  _ptr(nxt)))
        return nxt

    def step_rows(self, tokens, slots, positions, sample):
        """One step over arbitrary rows (token, cache slot, position); -> next ids after the rows `sample`."""
        tok = np.ascontiguousarray(tokens, dtype=np.int32)
        slot = np.ascontiguousarray(slots, dtype=np.int32)
        pos = np.ascontiguousarray(positions, dtype=np.int32)
        smp = np.ascontiguousarray(sample, dtype=np.int32)
        nxt = np.empty(smp.size, np.int32)
        _l.check(self.L.gptoss_engine_step_rows(self._h, tok.size, _ptr(tok), _ptr(slot), _ptr(pos), smp.size,
                                                _ptr(smp), _ptr(nxt)))
        return nxt

    def generate(self, prompts, max_seq_len, n_prompt=None, max_len=None):
        """Greedy generation; max_len (optional, per request) limits a request's total length."""
        prompts = np.ascontiguousarray(prompts, dtype=np.int32)
        n_req, stride = prompts.shape
        npr = np.full(n_req, stride, np.int32) if n_prompt is None else \
            np.ascontiguousarray(n_prompt, dtype=np.int32)
        out = np.zeros((n_req, max_seq_len + 1), np.int32)
        n = C.c_longlong(0)
        if max_len is None:
            _l.check(self.L.gptoss_engine_generate(self._h, _ptr(prompts),
                                                   _ptr(npr), stride, n_req,
                                                   max_seq_len, _ptr(out),
                                                   C.byref(n)))
        else:
            ml = np.ascontiguousarray(max_len, dtype=np.int32)
            _l.check(self.L.gptoss_engine_generate_ragged(self._h, _ptr(prompts),
                                                          _ptr(npr), stride, n_req,
                                                          max_seq_len, _ptr(ml),
                                                          _ptr(out), C.byref(n)))
        return out, int(n.value)

    def step_logits(self, tokens, slots, positions, want):
        """Run rows (token, cache slot, position) -> fp32 logits [len(want), vocab] of the rows `want`."""
        tok = np.ascontiguousarray(tokens, dtype=np.int32)
        slot = np.ascontiguousarray(slots, dtype=np.int32)
        pos = np.ascontiguousarray(positions, dtype=np.int32)
        want = np.ascontiguousarray(want, dtype=np.int32)
        out = np.empty((want.size, self.info.vocab), np.float32)
        _l.check(self.L.gptoss_engine_step_logits(self._h, tok.size, _ptr(tok), _ptr(slot), _ptr(pos), want.size,
                                                  _ptr(want), _ptr(out)))
        return out

    def acquire_slot(self):
        s = C.c_int()
        _l.check(self.L.gptoss_engine_slot_acquire(self._h, C.byref(s)))
        return s.value

    def release_slot(self, slot):
        _l.check(self.L.gptoss_engine_slot_release(self._h, int(slot)))

    def device_bytes(self):
        nb = C.c_size_t()
        _l.check(self.L.gptoss_engine_debug_views(self._h, None, None, C.byref(nb)))
        return nb.value

    def close(self):
        if getattr(self, "_h", None):
            self.L.gptoss_engine_destroy(self._h)
            self._h = None

    def __del__(self):
        self.close()
