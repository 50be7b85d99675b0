"""ctypes binding of the model registry (include/tl/models.h, part of libtl_qwen.so): a model opened by
its path - a GGUF file, or a folder with config.json and model.safetensors - that takes tokens in
portions of any size and generates greedily."""
import ctypes as C
import json
import os

import numpy as np

from . import qwen

i64, u32, cint, P = C.c_int64, C.c_uint32, C.c_int, C.c_void_p
_bound = False


def _load():
    global _bound
    L = qwen._load()
    if not _bound:
        sig = {
            "tlm_error": (C.c_char_p, []),
            "tlm_open": (P, [C.c_char_p, i64, i64, cint, cint]),
            "tlm_random": (P, [C.c_char_p, u32, i64, i64, i64, cint]),
            "tlm_close": (None, [P]),
            "tlm_architecture": (C.c_char_p, [P]),
            "tlm_vocab": (i64, [P]),
            "tlm_capacity": (i64, [P]),
            "tlm_pos": (i64, [P]),
            "tlm_reset": (None, [P]),
            "tlm_feed": (cint, [P, P, i64, P, i64, P]),
            "tlm_generate": (i64, [P, i64, i64, P]),
            "tlm_set_fused": (cint, [P, cint]),
            "tlm_layer_runs": (i64, [P]),
            "tlm_trace_chunk": (cint, [P, P, i64, P]),
            "tlm_capture_step": (cint, [P, i64, i64]),
            "tlm_replay_step": (cint, [P]),
            "tlm_eager_step": (cint, [P, i64, i64]),
            "tlm_stage_chunk": (cint, [P, P, i64]),
            "tlm_chunk_layers": (cint, [P, i64, i64]),
        }
        for name, (res, args) in sig.items():
            fn = getattr(L, name)
            fn.restype, fn.argtypes = res, args
        _bound = True
    return L


def _p(a):
    return a.ctypes.data_as(P)


class Model:
    """One sequence at a time on the GPU. No CPU fallback: opening raises when the backend is
    unavailable or the path holds no model this build knows."""

    def __init__(self, L, h):
        self.L, self.h = L, h
        if not h:
            raise RuntimeError(L.tlm_error().decode(errors="replace"))
        self.vocab, self.capacity = int(L.tlm_vocab(h)), int(L.tlm_capacity(h))

    @classmethod
    def open(cls, path, max_ctx=4096, chunk=512, exact=False, q4=False):
        """exact: prompt products exact in f32 instead of in two rounded terms per operand."""
        L = _load()
        return cls(L, L.tlm_open(os.fsencode(path), max_ctx, chunk, int(exact), int(q4)))

    @classmethod
    def random(cls, config, seed=1, rank=16, max_ctx=4096, chunk=512, exact=False):
        """A model of the given configuration (a dict with its "architecture") with seeded weights; rank: of
        Lusadra's decay inputs."""
        L = _load()
        return cls(L, L.tlm_random(json.dumps(config).encode(), seed, rank, max_ctx, chunk, int(exact)))

    @property
    def architecture(self):
        return self.L.tlm_architecture(self.h).decode()

    @property
    def pos(self):
        return int(self.L.tlm_pos(self.h))

    def reset(self):
        """Start a new sequence."""
        self.L.tlm_reset(self.h)

    def feed(self, tokens, want=()):
        """The sequence's next tokens; logits [len(want), vocab] of the listed places among them."""
        t, w = np.ascontiguousarray(tokens, np.int64), np.ascontiguousarray(want, np.int64)
        out = np.empty((len(w), self.vocab), np.float32)
        if self.L.tlm_feed(self.h, _p(t), len(t), _p(w), len(w), _p(out)) != 0:
            raise RuntimeError("feed declined (context full, token out of range, or a launch refused)")
        return out

    def generate(self, prompt, n):
        """Greedy continuation of the current sequence by `prompt`: n new tokens, the loop on the device."""
        first = int(np.argmax(self.feed(prompt, [len(prompt) - 1])[0]))
        out = np.empty(max(n - 1, 1), np.int32)
        done = int(self.L.tlm_generate(self.h, first, n - 1, _p(out))) if n > 1 else 0
        if n > 0 and done != n - 1:
            raise RuntimeError("generate: %d of %d tokens (context full, or the loop could not be recorded)" % (done + 1, n))
        return ([first] + [int(v) for v in out[:done]])[:n]

    # ---- launch forms, diagnostics, throughput (designs read from folders) -----------------------
    def set_fused(self, on):
        if self.L.tlm_set_fused(self.h, int(on)) != 0:
            raise RuntimeError("set_fused: not offered by this model")

    def trace_chunk(self, tokens, width):
        """The residual stream after every layer run of one chunk: [runs, tokens, width]."""
        t = np.ascontiguousarray(tokens, np.int64)
        out = np.empty((int(self.L.tlm_layer_runs(self.h)), len(t), width), np.float32)
        if self.L.tlm_trace_chunk(self.h, _p(t), len(t), _p(out)) != 0:
            raise RuntimeError("trace_chunk declined")
        return out

    def capture_step(self, token, pos):
        if self.L.tlm_capture_step(self.h, token, pos) != 0:
            raise RuntimeError("graph capture failed")

    def replay_step(self):
        if self.L.tlm_replay_step(self.h) != 0:
            raise RuntimeError("graph replay failed")

    def eager_step(self, token, pos):
        if self.L.tlm_eager_step(self.h, token, pos) != 0:
            raise RuntimeError("step declined")

    def stage_chunk(self, tokens):
        t = np.ascontiguousarray(tokens, np.int64)
        if self.L.tlm_stage_chunk(self.h, _p(t), len(t)) != 0:
            raise RuntimeError("stage_chunk declined")

    def chunk_layers(self, n, pos0):
        if self.L.tlm_chunk_layers(self.h, n, pos0) != 0:
            raise RuntimeError("chunk_layers declined")

    def flush(self):
        self.L.tlq_flush()

    def close(self):
        if self.h:
            self.L.tlm_close(self.h)
            self.h = None
