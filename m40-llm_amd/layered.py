"""ctypes view of layered decoders (m40host_model_open and what follows it in include/m40llm_host.h): models described by a
folder's config.json, served with a paged cache and a step function that takes any mixture of portions."""
from __future__ import annotations

import ctypes as C
import json

import numpy as np

from . import Context, host

ACT = {"bfloat16": 0, "float32": 1}


class ModelOptions(C.Structure):
    _fields_ = [(n, C.c_uint32) for n in ("act_dtype", "max_tokens", "max_sequences", "max_rows", "portion_form")]


class StepEntryC(C.Structure):
    _fields_ = [("sequence_id", C.c_uint32), ("n_tokens", C.c_uint32), ("n_want", C.c_uint32), ("tokens", C.c_void_p), ("want", C.c_void_p)]


class LayeredModel:
    """open(folder) or random(config dict); step([(sequence, tokens, want), ...]) -> logits [wanted][vocab]."""

    def __init__(self, ctx: Context, handle, vocab_width=None):
        self.ctx, self.H, self.h = ctx, host(), handle
        if not handle:
            raise RuntimeError(self.H.m40host_last_error().decode())
        self.vocab = self.H.m40host_model_vocab(handle)

    @classmethod
    def open(cls, ctx, folder, dtype="bfloat16", max_tokens=4096, max_sequences=4, max_rows=0, portion_form=0):
        o = ModelOptions(ACT[dtype], max_tokens, max_sequences, max_rows, portion_form)
        return cls(ctx, host().m40host_model_open(ctx.h, str(folder).encode(), C.byref(o)))

    @classmethod
    def random(cls, ctx, config: dict, seed=0, std=0.02, dtype="bfloat16", max_tokens=4096, max_sequences=4, max_rows=0, portion_form=0):
        o = ModelOptions(ACT[dtype], max_tokens, max_sequences, max_rows, portion_form)
        return cls(ctx, host().m40host_model_open_random(ctx.h, json.dumps(config).encode(), seed, std, C.byref(o)))

    def close(self):
        if getattr(self, "h", None):
            self.H.m40host_model_destroy(self.h)
            self.h = None

    def __del__(self):
        try:
            self.close()
        except Exception:
            pass

    def _ok(self, rc, what):
        if rc != 0:
            raise RuntimeError(f"{what} -> {rc}: {self.H.m40host_last_error().decode()}")

    def set_mode(self, mode: int):
        self._ok(self.H.m40host_model_set_mode(self.h, mode), "m40host_model_set_mode")

    def set_tie_guard(self, guard: float):
        self._ok(self.H.m40host_model_set_tie_guard(self.h, C.c_float(guard)), "m40host_model_set_tie_guard")

    def step(self, entries):
        keep, arr, n_want = [], (StepEntryC * len(entries))(), 0
        for i, (seq, tokens, want) in enumerate(entries):
            t = np.ascontiguousarray(tokens, dtype=np.uint32)
            w = np.ascontiguousarray(list(want), dtype=np.uint32)
            keep += [t, w]
            arr[i] = StepEntryC(seq, len(t), len(w), t.ctypes.data, w.ctypes.data if len(w) else None)
            n_want += len(w)
        out = np.empty((n_want, self.vocab), dtype=np.float32)
        self._ok(self.H.m40host_model_step(self.h, C.cast(arr, C.c_void_p), len(entries), out.ctypes.data if n_want else None), "m40host_model_step")
        return out

    def step_layers(self, seq, tokens, n_layers, width):
        t = np.ascontiguousarray(tokens, dtype=np.uint32)
        out = np.empty((n_layers, len(t), width), dtype=np.float32)
        e = StepEntryC(seq, len(t), 0, t.ctypes.data, None)
        self._ok(self.H.m40host_model_step_layers(self.h, C.byref(e), out.ctypes.data), "m40host_model_step_layers")
        return out

    def release(self, seq):
        self._ok(self.H.m40host_model_release(self.h, seq), "m40host_model_release")

    def assume_length(self, seq, tokens):
        self._ok(self.H.m40host_model_assume_length(self.h, seq, tokens), "m40host_model_assume_length")

    def length(self, seq):
        return self.H.m40host_model_length(self.h, seq)

    def free_pages(self):
        return self.H.m40host_model_free_pages(self.h)

    def decode_greedy(self, seq, prompt, n_gen, start_pos=0):
        p = np.ascontiguousarray(prompt, dtype=np.uint32)
        ids = np.zeros(len(p) + n_gen, dtype=np.uint32)
        gaps = np.zeros(max(n_gen, 1), dtype=np.float32)
        self._ok(self.H.m40host_model_decode_greedy(self.h, seq, p.ctypes.data_as(C.c_void_p), len(p), n_gen, start_pos,
                                                    ids.ctypes.data_as(C.c_void_p), gaps.ctypes.data_as(C.c_void_p)), "m40host_model_decode_greedy")
        return ids, gaps[:n_gen]

    def decode_batch_timed(self, seq_ids, kv_lens, first_tokens, warmup, steps):
        s, l, t = (np.ascontiguousarray(a, dtype=np.uint32) for a in (seq_ids, kv_lens, first_tokens))
        ids = np.zeros((len(s), warmup + steps), dtype=np.uint32)
        ms = C.c_double()
        self._ok(self.H.m40host_model_decode_batch_timed(self.h, s.ctypes.data_as(C.c_void_p), l.ctypes.data_as(C.c_void_p),
                                                         t.ctypes.data_as(C.c_void_p), len(s), warmup, steps,
                                                         ids.ctypes.data_as(C.c_void_p), C.byref(ms)), "m40host_model_decode_batch_timed")
        return ids, ms.value

    def last_timed_host_fallback(self):
        return bool(self.H.m40host_model_last_timed_host_fallback(self.h))
