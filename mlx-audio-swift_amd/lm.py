"""Language models described layer by layer in config.json ("architecture", "layers"): loading, the step function, batched generation.  The
device side is the token engine of libmi_speech (csrc/lm_engine.hip: rows, sampler, generate loop; csrc/lm_blocks.hip: layers and caches)."""
from __future__ import annotations

import ctypes as C
import json
import os
from dataclasses import dataclass, field, replace

import numpy as np

from . import _lib
from .codecs import _tensor_args
from .generation import AudioGenerationError, GenerateParameters, check, decode_audio_event, stream_events

MAX_BATCH = 64          # rows per engine call
COMPUTE = {"bfloat16": 0, "float32": 1}


@dataclass
class BlockModelConfiguration:
    """config.json of a model described layer by layer.  The engine parses and checks it (csrc/lm_blocks.hip); this mirror is for callers."""
    architecture: str
    width: int
    vocab: int
    layers: list = field(default_factory=list)
    norm: dict = field(default_factory=lambda: {"eps": 1e-6})
    logit_scale: float = 1.0
    logit_softcap: float = 0.0
    loop: dict | None = None            # {"start", "stop", "times"}: layers start .. stop - 1 run several times in a row

    @classmethod
    def from_dict(cls, d: dict) -> "BlockModelConfiguration":
        missing = [k for k in ("architecture", "width", "vocab", "layers") if k not in d]
        if missing:
            raise AudioGenerationError(3, f"config.json lacks {', '.join(missing)}")
        return cls(**{k: d[k] for k in cls.__dataclass_fields__ if k in d})

    def to_dict(self) -> dict:
        return {k: getattr(self, k) for k in self.__dataclass_fields__}


class BlockLanguageModel:
    """One handle = one model on one device, a batch of up to MAX_BATCH rows with their caches."""

    def __init__(self, config: BlockModelConfiguration, compute: str = "bfloat16", device: int = 0, _handle=None):
        self.configuration, self.compute, self.device = config, compute, device
        self.batch = 0
        self._h = _handle
        if self._h is None:
            h = C.c_void_p()
            check(_lib.lib().mis_lm_create(json.dumps(config.to_dict()).encode(), COMPUTE[compute], device, C.byref(h)))
            self._h = h

    # -- loading -----------------------------------------------------------------------------------
    @classmethod
    def from_model_directory(cls, model_dir: str, compute: str = "bfloat16", device: int = 0) -> "BlockLanguageModel":
        with open(os.path.join(model_dir, "config.json")) as f:
            cfg = BlockModelConfiguration.from_dict(json.load(f))
        h = C.c_void_p()
        check(_lib.lib().mis_lm_load(model_dir.encode(), COMPUTE[compute], device, C.byref(h)))
        return cls(cfg, compute, device, _handle=h)

    @classmethod
    def from_weights(cls, config, weights: dict, compute: str = "bfloat16", device: int = 0) -> "BlockLanguageModel":
        cfg = config if isinstance(config, BlockModelConfiguration) else BlockModelConfiguration.from_dict(config)
        m = cls(cfg, compute, device)
        for name, arr in weights.items():
            m.set_tensor(name, arr)
        m.finalize()
        return m

    @classmethod
    def synthetic(cls, config, compute: str = "bfloat16", device: int = 0, seed: int = 4321) -> "BlockLanguageModel":
        """Random weights generated on the device (benches)."""
        cfg = config if isinstance(config, BlockModelConfiguration) else BlockModelConfiguration.from_dict(config)
        m = cls(cfg, compute, device)
        check(_lib.lib().mis_tts_init_synthetic(m._h, seed))
        m.finalize()
        return m

    def set_tensor(self, name: str, arr):
        keep, ptr, dt, shape = _tensor_args(arr)
        sh = (C.c_int64 * len(shape))(*shape)
        check(_lib.lib().mis_tts_set_tensor(self._h, name.encode(), ptr, dt, sh, len(shape)))

    def finalize(self):
        check(_lib.lib().mis_tts_finalize(self._h))

    # -- step function -------------------------------------------------------------------------------
    @property
    def vocab_size(self) -> int:
        return int(_lib.lib().mis_lm_vocab_size(self._h))

    def reset(self, batch: int, max_context: int):
        """Empty caches for `batch` rows of up to max_context positions; what earlier rows held is given back."""
        check(_lib.lib().mis_lm_reset(self._h, int(batch), int(max_context)))
        self.batch = int(batch)

    def set_prefill_rows(self, rows: int):
        check(_lib.lib().mis_lm_set_prefill_rows(self._h, int(rows)))

    def extend(self, entries, want=None, return_residual: bool = False):
        """entries: [(batch row, token ids)] - the next tokens of each row; all entries run as one batch.  want: per entry the places among its
        tokens whose logits are returned (default: the last one).  -> float32 [wanted, vocab] in entry order (and the residual stream
        behind every layer, [layers, tokens, hidden])."""
        rows = np.asarray([r for r, _ in entries], np.int32)
        toks = [np.ascontiguousarray(t, dtype=np.int32).ravel() for _, t in entries]
        counts = np.asarray([len(t) for t in toks], np.int32)
        flat = np.ascontiguousarray(np.concatenate(toks))
        start = np.concatenate([[0], np.cumsum(counts)[:-1]])
        if want is None:
            want = [[len(t) - 1] for t in toks]
        for w, n in zip(want, counts):
            if any(i < 0 or i >= n for i in w):
                raise AudioGenerationError(3, "wanted place outside the entry's tokens")
        wv = np.asarray([int(s) + int(i) for s, w in zip(start, want) for i in w], np.int32)
        out = np.zeros((len(wv), self.vocab_size), np.float32)
        res = None
        if return_residual:
            res = np.zeros((int(_lib.lib().mis_lm_num_layers(self._h)), len(flat), int(_lib.lib().mis_lm_hidden_size(self._h))), np.float32)
        check(_lib.lib().mis_lm_extend(self._h, rows.ctypes.data, counts.ctypes.data, len(rows), flat.ctypes.data, wv.ctypes.data if len(wv) else None, len(wv),
                                       out.ctypes.data if len(wv) else None, res.ctypes.data if return_residual else None))
        return (out, res) if return_residual else out

    def prefill(self, prompt_rows, max_context: int = 0):
        """Ragged prompts from empty caches -> next-token logits [batch, vocab]; extend() / forward() continue behind them."""
        flat, lens = self._flatten(prompt_rows)
        out = np.zeros((len(lens), self.vocab_size), np.float32)
        check(_lib.lib().mis_lm_prefill(self._h, flat.ctypes.data, lens.ctypes.data, len(lens), int(max_context), out.ctypes.data, None))
        self.batch = len(lens)
        return out

    def forward(self, ids, active=None):
        """One token of every (active) row -> logits [batch, vocab]."""
        ids = np.ascontiguousarray(ids, dtype=np.int32)
        act = None if active is None else np.ascontiguousarray(active, dtype=np.uint8)
        out = np.zeros((len(ids), self.vocab_size), np.float32)
        check(_lib.lib().mis_lm_forward(self._h, ids.ctypes.data, act.ctypes.data if act is not None else None, out.ctypes.data))
        return out

    # -- generation ------------------------------------------------------------------------------------
    def generate_batch(self, prompt_rows, generation_parameters: GenerateParameters | None = None, stop_id: int = -1):
        """-> one int32 array of new ids per prompt (stop id included).  More than MAX_BATCH prompts run in slices (the sampler's random
        numbers are keyed by the global row index: slicing changes no row)."""
        gp = generation_parameters or GenerateParameters()
        if len(prompt_rows) > MAX_BATCH:
            out = []
            for i in range(0, len(prompt_rows), MAX_BATCH):
                out += self.generate_batch(prompt_rows[i:i + MAX_BATCH], replace(gp, row_offset=gp.row_offset + i), stop_id)
            return out
        flat, lens = self._flatten(prompt_rows)
        B = len(lens)
        gpc = gp.to_c()
        toks = np.zeros((B, gp.max_tokens), np.int32)
        n = np.zeros(B, np.int32)
        check(_lib.lib().mis_lm_generate(self._h, flat.ctypes.data, lens.ctypes.data, B, C.byref(gpc), int(stop_id), toks.ctypes.data, n.ctypes.data))
        self.batch = B
        return [toks[b, : n[b]].copy() for b in range(B)]

    def generate_stream_batch(self, prompt_rows, generation_parameters: GenerateParameters | None = None, stop_id: int = -1, cancel_flag=None):
        """TokenEvent per new id while the engine generates, then one InfoEvent per row."""
        gp = generation_parameters or GenerateParameters()
        flat, lens = self._flatten(prompt_rows)
        gpc = gp.to_c()

        def start(cbf, flag_addr):
            return _lib.lib().mis_lm_generate_stream(self._h, flat.ctypes.data, lens.ctypes.data, len(lens), C.byref(gpc), int(stop_id), cbf, None, flag_addr)
        yield from stream_events(start, decode_audio_event, cancel_flag)

    def last_timing(self) -> dict:
        t = _lib.TimingC()
        check(_lib.lib().mis_tts_last_timing(self._h, C.byref(t)))
        return {k: getattr(t, k) for k, _ in t._fields_}

    @staticmethod
    def _flatten(rows):
        rows = [np.ascontiguousarray(r, dtype=np.int32).ravel() for r in rows]
        if not rows:
            raise AudioGenerationError(3, "empty batch")
        return np.ascontiguousarray(np.concatenate(rows)), np.asarray([len(r) for r in rows], np.int32)

    def close(self):
        if self._h is not None:
            _lib.lib().mis_tts_destroy(self._h)
            self._h = None

    def __del__(self):
        try:
            self.close()
        except Exception:
            pass
