"""Model class by config.json, the counterpart of `TTS.loadModel` (Sources/MLXAudioTTS/TTSModel.swift:104-219) for local directories:
"architecture" names a model described layer by layer, "model_type" (or its absence) the Llama family."""
from __future__ import annotations

import json
import os

from .generation import AudioGenerationError
from .lm import BlockLanguageModel
from .tts import LlamaTTSModel

ARCHITECTURES = {"Rugunex": BlockLanguageModel, "Vamunex": BlockLanguageModel}
MODEL_TYPES = {"llama": LlamaTTSModel, "qwen3": LlamaTTSModel, "orpheus": LlamaTTSModel}
# classes whose engine has a true 32-bit mode
FLOAT32 = {BlockLanguageModel}


def model_class(config: dict):
    arch = config.get("architecture")
    if arch is not None:
        if arch not in ARCHITECTURES:
            raise AudioGenerationError(3, f"unknown architecture {arch!r} (known: {', '.join(sorted(ARCHITECTURES))})")
        return ARCHITECTURES[arch]
    mt = str(config.get("model_type", "llama")).lower()
    for name, cls in MODEL_TYPES.items():
        if name in mt:
            return cls
    raise AudioGenerationError(3, f"unknown model_type {mt!r}")


def load_model(model_dir: str, compute: str = "bfloat16", device: int = 0, **kw):
    with open(os.path.join(model_dir, "config.json")) as f:
        cls = model_class(json.load(f))
    if cls in FLOAT32:
        return cls.from_model_directory(model_dir, compute=compute, device=device, **kw)
    if compute != "bfloat16":
        raise AudioGenerationError(3, f"{cls.__name__} runs in bfloat16 only")
    return cls.from_model_directory(model_dir, device=device, **kw)
