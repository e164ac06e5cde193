"""Model configurations (public architecture hyper-parameters; weights are random-init or
loaded from safetensors).  The reference calls hosted models instead
(gpt-4o-mini: apps/brain/src/llm.ts:9; Deepgram nova-3: apps/voice/src/server.ts:106); the
north star names these on-node replacements.
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass, field, replace
from typing import Optional


@dataclass(frozen=True)
class LlamaConfig:
    name: str = "llama3-8b"
    vocab_size: int = 128256
    hidden: int = 4096
    n_layers: int = 32
    n_heads: int = 32
    n_kv_heads: int = 8
    head_dim: int = 128
    ffn: int = 14336
    rope_theta: float = 500000.0
    rms_eps: float = 1e-5
    max_pos: int = 8192
    tie_embeddings: bool = False
    bos_id: int = 128000
    eos_ids: tuple = (128001, 128009)
    init_std: float = 0.02


@dataclass(frozen=True)
class GPT2Config:
    name: str = "gpt2-small"
    vocab_size: int = 50257
    hidden: int = 768
    n_layers: int = 12
    n_heads: int = 12
    ffn: int = 3072
    # n_positions is 1024 in the public config; the intent prompt is ~1.1k tokens, so the
    # CPU config runs with 2048 learned positions.
    max_pos: int = 2048
    ln_eps: float = 1e-5
    bos_id: int = 50256
    eos_ids: tuple = (50256,)
    init_std: float = 0.02

    @property
    def head_dim(self) -> int:
        return self.hidden // self.n_heads

    @property
    def n_kv_heads(self) -> int:
        return self.n_heads


@dataclass(frozen=True)
class WhisperConfig:
    name: str = "whisper-tiny"
    n_mels: int = 80
    n_audio_ctx: int = 1500
    d_model: int = 384
    n_heads: int = 6
    n_enc_layers: int = 4
    n_dec_layers: int = 4
    n_text_ctx: int = 448
    vocab_size: int = 51865
    ln_eps: float = 1e-5
    init_std: float = 0.02
    # special tokens (multilingual layout)
    eot: int = 50257
    sot: int = 50258
    lang_en: int = 50259
    transcribe: int = 50359
    no_timestamps: int = 50363

    @property
    def head_dim(self) -> int:
        return self.d_model // self.n_heads

    @property
    def ffn(self) -> int:
        return 4 * self.d_model


@dataclass(frozen=True)
class TalkAttentionConfig:
    """Windowed grouped-query attention with kept first keys, partial rotation, softmax weights mixed
    across the query heads and an output gate per head."""
    heads: int
    kv_heads: int
    dim: int                 # query / key size of a head
    vdim: int                # value size of a head
    scale: float
    window: int              # a position sees the last ``window`` positions (itself included) ...
    keep_first: int          # ... and the first ``keep_first`` of the sequence
    rot_base: float
    rot_dims: int            # rotated dimensions of every query / key head (the first ones)


@dataclass(frozen=True)
class MinGRUConfig:
    width: int


@dataclass(frozen=True)
class ParallelLayerConfig:
    """One layer: two mixers side by side, and a feed-forward (0: none), all reading one normed input."""
    left: TalkAttentionConfig
    right: MinGRUConfig
    left_scale: float = 1.0
    right_scale: float = 1.0
    ffn: int = 0


@dataclass(frozen=True)
class KabanexConfig:
    name: str
    vocab_size: int
    hidden: int
    layers: tuple            # of ParallelLayerConfig, in order (sizes may differ from layer to layer)
    norm_eps: float = 1e-5
    max_pos: int = 8192      # rotation table length to start with (it grows with the engine's contexts)
    bos_id: int = 0
    eos_ids: tuple = ()
    init_std: float = 0.02

    @property
    def n_layers(self) -> int:
        return len(self.layers)

    @staticmethod
    def from_json(j: dict, name: str = "kabanex") -> "KabanexConfig":
        """The checkpoint's config.json.  A layer, feed-forward or norm kind this design does not have
        is an error, never ignored."""
        layers = []
        for i, L in enumerate(j["layers"]):
            if L["type"] != "parallel":
                raise ValueError(f"layer {i}: unknown mixer type {L['type']!r}")
            m, mlp = L["mixer"], L.get("mlp")
            if mlp is not None and mlp["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
            a = m["left"]
            if a["heads"] % a["kv_heads"] or a["rot"]["dims"] % 2 or not 0 < a["rot"]["dims"] <= a["dim"]:
                raise ValueError(f"layer {i}: head counts or rotated dimensions do not fit")
            if a["mask"]["size"] < 1 or a["mask"]["keep_first"] < 0:
                raise ValueError(f"layer {i}: window size must be positive, kept keys not negative")
            layers.append(ParallelLayerConfig(
                left=TalkAttentionConfig(heads=a["heads"], kv_heads=a["kv_heads"], dim=a["dim"], vdim=a["vdim"],
                                         scale=float(a["scale"]), window=a["mask"]["size"],
                                         keep_first=a["mask"]["keep_first"], rot_base=float(a["rot"]["base"]),
                                         rot_dims=a["rot"]["dims"]),
                right=MinGRUConfig(width=m["right"]["width"]), left_scale=float(m["left_scale"]),
                right_scale=float(m["right_scale"]), ffn=mlp["ff"] if mlp is not None else 0))
        return KabanexConfig(name=name, vocab_size=j["vocab"], hidden=j["width"], layers=tuple(layers),
                             norm_eps=float(j["norm"]["eps"]))


def kabanex_stack(name: str, *, vocab: int, hidden: int, n_layers: int, heads: int, kv_heads: int, dim: int, vdim: int,
                  window: int, keep_first: int, width: int, ffn: int, rot_dims: Optional[int] = None,
                  rot_base: float = 500000.0, **kw) -> KabanexConfig:
    """A uniform stack (presets, benchmarks)."""
    L = ParallelLayerConfig(
        left=TalkAttentionConfig(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=dim ** -0.5, window=window,
                                 keep_first=keep_first, rot_base=rot_base, rot_dims=rot_dims or dim // 2),
        right=MinGRUConfig(width=width), ffn=ffn)
    return KabanexConfig(name=name, vocab_size=vocab, hidden=hidden, layers=(L,) * n_layers, **kw)


@dataclass(frozen=True)
class RgLruConfig:
    """Gated branch beside a short causal convolution and a real-gated linear recurrence, whose gates are
    block-diagonal in the recurrence's channels."""
    width: int
    blocks: int
    conv: int                # taps

    @property
    def block(self) -> int:
        return self.width // self.blocks


@dataclass(frozen=True)
class LatentAttentionConfig:
    """Attention whose keys and values are projections of one cached latent, with a shared rotated key part,
    a softmax sink per head and an output gate per element."""
    heads: int
    dim: int                 # unrotated query / key size of a head
    rot_dim: int             # rotated query / key size of a head
    vdim: int
    kv_rank: int
    scale: float
    rot_base: float
    kv_from: Optional[int] = None    # the layer whose cached latent this one reads (None: its own)


@dataclass(frozen=True)
class DenseFFConfig:
    ff: int


@dataclass(frozen=True)
class MoEConfig:
    """``experts`` feed-forwards of size ff, of which a token uses the ``top`` with the largest sigmoid scores;
    the score scales the expert's input."""
    experts: int
    top: int
    ff: int


@dataclass(frozen=True)
class SerialLayerConfig:
    """A mixer, then a feed-forward (None: none), each between two norms."""
    mixer: object            # RgLruConfig | LatentAttentionConfig
    mlp: object = None       # DenseFFConfig | MoEConfig | None


@dataclass(frozen=True)
class RipupelConfig:
    name: str
    vocab_size: int
    hidden: int
    layers: tuple            # of SerialLayerConfig, in order (sizes may differ from layer to layer)
    embed_scale: float = 1.0
    norm_eps: float = 1e-6
    max_pos: int = 8192      # rotation table length to start with (it grows with the engine's contexts)
    bos_id: int = 0
    eos_ids: tuple = ()
    init_std: float = 0.02

    @property
    def n_layers(self) -> int:
        return len(self.layers)

    @staticmethod
    def from_json(j: dict, name: str = "ripupel") -> "RipupelConfig":
        """The checkpoint's config.json.  A mixer or feed-forward kind this design does not have is an error,
        never ignored."""
        layers = []
        for i, L in enumerate(j["layers"]):
            m, mlp = L["mixer"], L.get("mlp")
            if L["type"] == "rglru":
                mixer = RgLruConfig(width=m["width"], blocks=m["blocks"], conv=m["conv"])
                if mixer.blocks < 1 or mixer.width % mixer.blocks or mixer.conv < 1:
                    raise ValueError(f"layer {i}: recurrence width, blocks or convolution taps do not fit")
            elif L["type"] == "latent_attention":
                mixer = LatentAttentionConfig(heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"], vdim=m["vdim"],
                                              kv_rank=m["kv_rank"], scale=float(m["scale"]), rot_base=float(m["rot"]["base"]),
                                              kv_from=m.get("kv_from"))
                if mixer.rot_dim < 2 or mixer.rot_dim % 2 or m["rot"]["dims"] != mixer.rot_dim:
                    raise ValueError(f"layer {i}: rotated dimensions do not fit")
                if mixer.kv_from is not None:
                    src = layers[mixer.kv_from].mixer if 0 <= mixer.kv_from < i else None
                    if not isinstance(src, LatentAttentionConfig) or src.kv_from is not None or \
                            (src.kv_rank, src.rot_dim, src.rot_base) != (mixer.kv_rank, mixer.rot_dim, mixer.rot_base):
                        raise ValueError(f"layer {i}: layer {mixer.kv_from} has no latent it could share")
            else:
                raise ValueError(f"layer {i}: unknown mixer type {L['type']!r}")
            if mlp is None:
                ff = None
            elif mlp["kind"] == "dense":
                ff = DenseFFConfig(ff=mlp["ff"])
            elif mlp["kind"] == "moe":
                ff = MoEConfig(experts=mlp["router"]["experts"], top=mlp["router"]["top"], ff=mlp["expert"]["ff"])
                if not 1 <= ff.top <= ff.experts:
                    raise ValueError(f"layer {i}: {ff.top} of {ff.experts} experts")
            else:
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
            layers.append(SerialLayerConfig(mixer=mixer, mlp=ff))
        return RipupelConfig(name=name, vocab_size=j["vocab"], hidden=j["width"], layers=tuple(layers),
                             embed_scale=float(j["embedding"]["scale"]), norm_eps=float(j["norm"]["eps"]))


def ripupel_stack(name: str, *, vocab: int, hidden: int, n_layers: int, heads: int, dim: int, rot_dim: int, vdim: int,
                  kv_rank: int, width: int, blocks: int, ffn: int, experts: int, top: int, expert_ff: int, conv: int = 4,
                  rot_base: float = 500000.0, **kw) -> RipupelConfig:
    """Recurrent layers with a dense feed-forward and attention layers with routed experts in turn, every second
    attention layer on the latent of the one before (presets, benchmarks)."""
    layers = []
    for i in range(n_layers):
        if i % 2 == 0:
            layers.append(SerialLayerConfig(RgLruConfig(width=width, blocks=blocks, conv=conv), DenseFFConfig(ffn)))
        else:
            layers.append(SerialLayerConfig(
                LatentAttentionConfig(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank,
                                      scale=(dim + rot_dim) ** -0.5, rot_base=rot_base, kv_from=i - 2 if i % 4 == 3 else None),
                MoEConfig(experts=experts, top=top, ff=expert_ff)))
    return RipupelConfig(name=name, vocab_size=vocab, hidden=hidden, layers=tuple(layers), **kw)


LLAMA_PRESETS = {
    "llama3-8b": LlamaConfig(),
    "llama3-70b": LlamaConfig(name="llama3-70b", hidden=8192, n_layers=80, n_heads=64, n_kv_heads=8, ffn=28672),
    "llama3.2-1b": LlamaConfig(name="llama3.2-1b", hidden=2048, n_layers=16, n_heads=32, n_kv_heads=8, head_dim=64,
                               ffn=8192, tie_embeddings=True),
    # small shapes for CPU tests (vocab kept at the real tokenizer size so the grammar works)
    "llama-tiny": LlamaConfig(name="llama-tiny", hidden=256, n_layers=2, n_heads=4, n_kv_heads=2, head_dim=64,
                              ffn=512, max_pos=4096),
}

GPT2_PRESETS = {
    "gpt2-small": GPT2Config(),
    "gpt2-tiny": GPT2Config(name="gpt2-tiny", hidden=128, n_layers=2, n_heads=2, ffn=512),
}

WHISPER_PRESETS = {
    "whisper-tiny": WhisperConfig(),
    "whisper-base": WhisperConfig(name="whisper-base", d_model=512, n_heads=8, n_enc_layers=6, n_dec_layers=6),
    "whisper-small": WhisperConfig(name="whisper-small", d_model=768, n_heads=12, n_enc_layers=12, n_dec_layers=12),
    "whisper-large-v3": WhisperConfig(name="whisper-large-v3", n_mels=128, d_model=1280, n_heads=20, n_enc_layers=32,
                                      n_dec_layers=32, vocab_size=51866, lang_en=50259, transcribe=50360,
                                      no_timestamps=50364),
    "whisper-test": WhisperConfig(name="whisper-test", d_model=128, n_heads=2, n_enc_layers=2, n_dec_layers=2),
}


KABANEX_PRESETS = {
    # Llama-3.2-1B-sized layers (bench.py --design): its residual width, feed-forward and vocabulary
    "kabanex-1b": kabanex_stack("kabanex-1b", vocab=128256, hidden=2048, n_layers=16, heads=16, kv_heads=4, dim=128, vdim=128,
                                window=1024, keep_first=4, width=2048, ffn=8192, bos_id=128000, eos_ids=(128001, 128009)),
    # small shapes for tests (vocab kept at the real tokenizer size so the grammar works)
    "kabanex-tiny": kabanex_stack("kabanex-tiny", vocab=128256, hidden=192, n_layers=2, heads=6, kv_heads=2, dim=32, vdim=48,
                                  window=640, keep_first=3, width=160, ffn=384, bos_id=128000,
                                  eos_ids=(128001, 128009)),
}


RIPUPEL_PRESETS = {
    # Llama-3.2-1B-sized layers (bench.py --design): its residual width, feed-forward and vocabulary
    "ripupel-1b": ripupel_stack("ripupel-1b", vocab=128256, hidden=2048, n_layers=16, heads=16, dim=128, rot_dim=64, vdim=128,
                                kv_rank=512, width=2048, blocks=16, ffn=8192, experts=32, top=4, expert_ff=1024, bos_id=128000,
                                eos_ids=(128001, 128009)),
    # small shapes for tests (vocab kept at the real tokenizer size so the grammar works)
    "ripupel-tiny": ripupel_stack("ripupel-tiny", vocab=128256, hidden=192, n_layers=4, heads=3, dim=32, rot_dim=16, vdim=48,
                                  kv_rank=64, width=192, blocks=3, ffn=256, experts=6, top=2, expert_ff=64, bos_id=128000,
                                  eos_ids=(128001, 128009)),
}


def _llama_from_json(j: dict, name: str) -> LlamaConfig:
    hd = j.get("head_dim") or j["hidden_size"] // j["num_attention_heads"]
    return LlamaConfig(name=name, vocab_size=j["vocab_size"], hidden=j["hidden_size"], n_layers=j["num_hidden_layers"],
                       n_heads=j["num_attention_heads"], n_kv_heads=j["num_key_value_heads"], head_dim=hd,
                       ffn=j["intermediate_size"], rope_theta=j["rope_theta"], rms_eps=j["rms_norm_eps"],
                       tie_embeddings=bool(j.get("tie_word_embeddings", False)))


# config.json "architecture" (or the first of "architectures") -> configuration reader
ARCHITECTURES = {
    "Kabanex": KabanexConfig.from_json,
    "LlamaForCausalLM": _llama_from_json,
    "Ripupel": RipupelConfig.from_json,
}


def config_from_dir(path: str):
    """The configuration of a checkpoint folder, by its config.json."""
    with open(os.path.join(path, "config.json"), encoding="utf-8") as fh:
        j = json.load(fh)
    arch = j.get("architecture") or (j.get("architectures") or [None])[0]
    if arch not in ARCHITECTURES:
        raise KeyError(f"unknown model architecture {arch!r} (known: {', '.join(sorted(ARCHITECTURES))})")
    return ARCHITECTURES[arch](j, os.path.basename(os.path.normpath(path)))


def get_config(name: str):
    """A preset by name, or the configuration of a checkpoint folder."""
    if os.path.isfile(os.path.join(name, "config.json")):
        return config_from_dir(name)
    for table in (LLAMA_PRESETS, GPT2_PRESETS, KABANEX_PRESETS, RIPUPEL_PRESETS, WHISPER_PRESETS):
        if name in table:
            return table[name]
    raise KeyError(f"unknown model preset {name!r}")
