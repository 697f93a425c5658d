from . import dafutar, dolezen, katenex, qwen2, sozavik, vagozen  # register Dafutar, Dolezen, Katenex, Qwen2ForCausalLM, Sozavik and Vagozen

__all__ = ["dafutar", "dolezen", "katenex", "qwen2", "sozavik", "vagozen"]
