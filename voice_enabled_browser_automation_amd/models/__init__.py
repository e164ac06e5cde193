"""Model classes and their registry (configuration type -> class)."""


def model_class(cfg):
    """The model class that runs a configuration."""
    from .config import GPT2Config, KabanexConfig, LlamaConfig, RipupelConfig

    if isinstance(cfg, LlamaConfig):
        from .llama import LlamaModel

        return LlamaModel
    if isinstance(cfg, GPT2Config):
        from .gpt2 import GPT2Model

        return GPT2Model
    if isinstance(cfg, KabanexConfig):
        from .kabanex import KabanexModel

        return KabanexModel
    if isinstance(cfg, RipupelConfig):
        from .ripupel import RipupelModel

        return RipupelModel
    raise TypeError(f"no language model class for {type(cfg).__name__}")
