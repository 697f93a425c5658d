from . import dafutar, dolezen, dubesun, katenex, qwen2, sozavik, vagozen  # register Dafutar, Dolezen, Dubesun, Katenex, Qwen2ForCausalLM, Sozavik and Vagozen

__all__ = ["dafutar", "dolezen", "dubesun", "katenex", "qwen2", "sozavik", "vagozen"]
