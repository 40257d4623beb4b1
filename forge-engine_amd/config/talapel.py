"""Configuration of the Talapel decoder, from its config.json keys.

config.json names the design under ``architecture`` and gives the vocabulary (``vocab``), the model
width (``width``), the norms' epsilon (``norm.eps``), a factor on the embedding
(``embedding.scale``), the list ``layers`` and optionally ``loop`` (``start``, ``stop``, ``times``: that run of
layers is passed through so many times).  Each layer entry has a ``type`` (which mixer: ``parallel`` or
``retention``), the mixer's sizes and constants (``mixer``) and its feed-forward (``mlp``: ``kind`` ``dense``
with ``ff``; ``kind`` ``moe`` with ``router.experts``, ``router.top``, ``expert.ff``; or null for none).  Mixer keys:
``parallel``: ``left`` (attention: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``softcap`` (absent: none),
``q_temp.coef``, ``q_temp.every`` (absent: none)), ``right`` (state-space recurrence: ``heads``, ``vdim``, ``state``,
``groups``, ``conv``, ``norm_groups``), ``left_scale``, ``right_scale``; ``retention``: ``heads``, ``dim``, ``vdim``,
``decay`` (one number a head), ``rot.dims``, ``rot.base``.  Every size and constant of a model comes from here;
nothing is pinned to one checkpoint.
"""

from __future__ import annotations

import json
from dataclasses import dataclass
from typing import Any, ClassVar

from .model import ConfigError, KeyReader, ModelConfig

MIXER_TYPES = ("parallel", "retention")
MLP_KINDS = ("dense", "moe")


def section(raw: dict, key: str, where: str) -> dict:
    value = raw.get(key)
    if not isinstance(value, dict):
        raise ConfigError(f"{where} needs an object '{key}'")
    return value


def _finite(raw: dict, key: str, where: str) -> float:
    """A number of any sign."""
    value = raw.get(key)
    if isinstance(value, bool) or not isinstance(value, (int, float)) or value != value or abs(value) == float("inf"):
        raise ConfigError(f"{where}: '{key}' must be a finite number, got {value!r}")
    return float(value)


def _check_attention(raw: dict, where: str) -> None:
    read = KeyReader(raw)
    heads, kv_heads = read.integer("heads"), read.integer("kv_heads")
    if heads % kv_heads:
        raise ConfigError(f"{where}: heads ({heads}) must be a multiple of kv_heads ({kv_heads})")
    for key in ("dim", "vdim"):
        if read.integer(key) > 256:
            raise ConfigError(f"{where}: '{key}' of up to 256")
    _finite(raw, "scale", where)
    if raw.get("softcap") is not None:
        read.number("softcap")
    if raw.get("q_temp") is not None:
        temp = section(raw, "q_temp", where)
        _finite(temp, "coef", where)
        KeyReader(temp).number("every")


def check_state_space(raw: dict, where: str) -> None:
    read = KeyReader(raw)
    heads, vdim, groups, parts = (read.integer(key) for key in ("heads", "vdim", "groups", "norm_groups"))
    if read.integer("state") > 256:
        raise ConfigError(f"{where}: up to 256 states")
    if read.integer("conv") > 8:
        raise ConfigError(f"{where}: a short convolution of up to 8 taps")
    if heads % groups:
        raise ConfigError(f"{where}: heads ({heads}) must be a multiple of groups ({groups})")
    if heads * vdim % parts:
        raise ConfigError(f"{where}: heads x vdim ({heads * vdim}) must be a multiple of norm_groups ({parts})")


def _check_retention(raw: dict, where: str) -> None:
    read = KeyReader(raw)
    heads, dim = read.integer("heads"), read.integer("dim")
    read.integer("vdim")
    if dim > 256:
        raise ConfigError(f"{where}: 'dim' of up to 256")
    decay = raw.get("decay")
    if (not isinstance(decay, list) or len(decay) != heads
            or not all(isinstance(d, (int, float)) and not isinstance(d, bool) and 0.0 < d < float("inf") for d in decay)):
        raise ConfigError(f"{where}: 'decay' must list {heads} positive numbers, got {decay!r}")
    rot = section(raw, "rot", where)
    dims = KeyReader(rot).integer("dims", minimum=2)
    KeyReader(rot).number("base")
    if dims % 2 or dims > dim:
        raise ConfigError(f"{where}: rot.dims ({dims}) must be even and at most dim ({dim})")


def _check_mlp(mlp: Any, where: str) -> None:
    if mlp is None:
        return
    if not isinstance(mlp, dict) or mlp.get("kind") not in MLP_KINDS:
        raise ConfigError(f"{where}: mlp must be null or of kind {' / '.join(MLP_KINDS)}")
    if mlp["kind"] == "dense":
        KeyReader(mlp).integer("ff")
        return
    KeyReader(section(mlp, "expert", where)).integer("ff")
    router = KeyReader(section(mlp, "router", where))
    experts, top = router.integer("experts"), router.integer("top")
    if top > experts:
        raise ConfigError(f"{where}: router.top ({top}) exceeds router.experts ({experts})")
    if top > 16 or experts > 1024:
        raise ConfigError(f"{where}: up to 16 experts a token out of up to 1,024")


def _check_layer(layer: Any, where: str) -> None:
    if not isinstance(layer, dict):
        raise ConfigError(f"{where} must be an object")
    kind = layer.get("type")
    if kind not in MIXER_TYPES:
        raise ConfigError(f"{where}: unknown mixer type {kind!r} (known: {', '.join(MIXER_TYPES)})")
    mixer = section(layer, "mixer", where)
    if kind == "retention":
        _check_retention(mixer, f"{where}.mixer")
    else:
        _check_attention(section(mixer, "left", where), f"{where}.mixer.left")
        check_state_space(section(mixer, "right", where), f"{where}.mixer.right")
        for key in ("left_scale", "right_scale"):
            _finite(mixer, key, f"{where}.mixer")
    _check_mlp(layer.get("mlp"), f"{where}.mlp")


def read_loop(raw: Any, layers: int) -> tuple[int, int, int] | None:
    if raw is None:
        return None
    if not isinstance(raw, dict):
        raise ConfigError("'loop' must be an object")
    read = KeyReader(raw)
    start, stop, times = read.integer("start", minimum=0), read.integer("stop"), read.integer("times")
    if not start < stop <= layers:
        raise ConfigError(f"loop: layers {start} .. {stop - 1} are not a run of the {layers} layers")
    return start, stop, times


@dataclass(frozen=True)
class TalapelConfig(ModelConfig):
    vocab: int
    width: int
    norm_eps: float
    layers_json: str                              # the list ``layers`` as JSON text (a frozen, hashable form)
    loop: tuple[int, int, int] | None = None      # (start, stop, times)
    embedding_scale: float = 1.0
    eos_token_id: int | None = None

    architecture: ClassVar[str] = "Talapel"

    @property
    def layers(self) -> list[dict]:
        return json.loads(self.layers_json)

    @classmethod
    def from_dict(cls, raw: dict[str, Any]) -> "TalapelConfig":
        read = KeyReader(raw)
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json must list the model's layers under 'layers'")
        for index, layer in enumerate(layers):
            _check_layer(layer, f"layers[{index}]")
        embedding = raw.get("embedding")
        scale = 1.0 if embedding is None else _finite(section(raw, "embedding", "config.json"), "scale", "embedding")
        eos = raw.get("eos_token_id")
        if eos is not None and (isinstance(eos, bool) or not isinstance(eos, int)):
            raise ConfigError(f"'eos_token_id' must be an integer, got {eos!r}")
        return cls(vocab=read.integer("vocab"), width=read.integer("width"),
                   norm_eps=KeyReader(section(raw, "norm", "config.json")).number("eps"),
                   layers_json=json.dumps(layers, sort_keys=True), loop=read_loop(raw.get("loop"), len(layers)),
                   embedding_scale=scale, eos_token_id=eos)

    def to_dict(self) -> dict[str, Any]:
        data = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
                "norm": {"eps": self.norm_eps}, "embedding": {"scale": self.embedding_scale}, "layers": self.layers}
        if self.loop is not None:
            data["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        if self.eos_token_id is not None:
            data["eos_token_id"] = self.eos_token_id
        return data
