"""Configuration of the Budanex decoder, from its config.json keys.

config.json names the design under ``architecture`` and gives the vocabulary (``vocab``), the model
width (``width``), the norms' epsilon (``norm.eps``), optionally a soft cap on the logits (``logit_softcap``), the list
``layers`` and optionally ``loop`` (``start``, ``stop``, ``times``: that run of layers is passed through so many
times).  Each layer entry has a ``type`` (which mixer: ``attention``, ``mamba2`` or ``latent_attention``), the mixer's
sizes and constants (``mixer``) and its feed-forward (``mlp``: ``kind`` ``dense`` with ``ff``; or null for none).
Mixer keys: ``attention``: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``softcap`` (absent: none), ``rot.dims``,
``rot.base``; ``mamba2``: ``heads``, ``vdim``, ``state``, ``groups``, ``conv``, ``norm_groups``; ``latent_attention``:
``heads``, ``dim``, ``rot_dim``, ``vdim``, ``kv_rank``, ``scale``, ``mask.size`` (the sliding window; absent: every earlier
token is seen), ``rot.dims``, ``rot.base`` and ``rot.scaling`` (``factor``, ``original``, ``fast``, ``slow``; absent: plain
frequencies).  Every size and constant of a model comes from here; nothing is pinned to one checkpoint.
"""

from __future__ import annotations

import json
from dataclasses import dataclass
from typing import Any, ClassVar

from .model import ConfigError, KeyReader, ModelConfig
from .talapel import check_state_space, read_loop, section

MLP_KINDS = ("dense",)


def _check_rotation(raw: dict, most: int, where: str) -> None:
    rot = section(raw, "rot", where)
    read = KeyReader(rot)
    dims = read.integer("dims", minimum=2)
    if not read.number("base") > 1.0:
        raise ConfigError(f"{where}: rot.base must be above 1")
    if dims % 2 or dims > most:
        raise ConfigError(f"{where}: rot.dims ({dims}) must be even and at most {most}")
    if rot.get("scaling") is not None:
        scaling = KeyReader(section(rot, "scaling", where))
        for key in ("factor", "original", "fast", "slow"):
            scaling.number(key)


def _check_attention(raw: dict, where: str) -> None:
    read = KeyReader(raw)
    heads, kv_heads = read.integer("heads"), read.integer("kv_heads")
    if heads % kv_heads:
        raise ConfigError(f"{where}: heads ({heads}) must be a multiple of kv_heads ({kv_heads})")
    dim = read.integer("dim", minimum=2)
    if dim > 256 or dim % 2 or read.integer("vdim") > 256:
        raise ConfigError(f"{where}: an even 'dim' and a 'vdim' of up to 256")
    read.number("scale")
    if raw.get("softcap") is not None:
        read.number("softcap")
    _check_rotation(raw, dim, where)


def _check_latent(raw: dict, where: str) -> None:
    read = KeyReader(raw)
    for key in ("heads", "dim", "vdim"):
        read.integer(key)
    if read.integer("kv_rank") > 512 or read.integer("rot_dim", minimum=2) > 128:
        raise ConfigError(f"{where}: 'kv_rank' of up to 512 and 'rot_dim' of up to 128")
    read.number("scale")
    if raw.get("mask") is not None:
        KeyReader(section(raw, "mask", where)).integer("size")
    _check_rotation(raw, raw["rot_dim"], where)


CHECKS = {"attention": _check_attention, "mamba2": check_state_space, "latent_attention": _check_latent}


def _check_layer(layer: Any, where: str) -> None:
    if not isinstance(layer, dict):
        raise ConfigError(f"{where} must be an object")
    kind = layer.get("type")
    if kind not in CHECKS:
        raise ConfigError(f"{where}: unknown mixer type {kind!r} (known: {', '.join(CHECKS)})")
    CHECKS[kind](section(layer, "mixer", where), f"{where}.mixer")
    mlp = layer.get("mlp")
    if mlp is None:
        return
    if not isinstance(mlp, dict) or mlp.get("kind") not in MLP_KINDS:
        raise ConfigError(f"{where}: mlp must be null or of kind {' / '.join(MLP_KINDS)}")
    KeyReader(mlp).integer("ff")


@dataclass(frozen=True)
class BudanexConfig(ModelConfig):
    vocab: int
    width: int
    norm_eps: float
    layers_json: str                              # the list ``layers`` as JSON text (a frozen, hashable form)
    loop: tuple[int, int, int] | None = None      # (start, stop, times)
    logit_softcap: float | None = None
    eos_token_id: int | None = None

    architecture: ClassVar[str] = "Budanex"

    @property
    def layers(self) -> list[dict]:
        return json.loads(self.layers_json)

    @classmethod
    def from_dict(cls, raw: dict[str, Any]) -> "BudanexConfig":
        read = KeyReader(raw)
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json must list the model's layers under 'layers'")
        for index, layer in enumerate(layers):
            _check_layer(layer, f"layers[{index}]")
        eos = raw.get("eos_token_id")
        if eos is not None and (isinstance(eos, bool) or not isinstance(eos, int)):
            raise ConfigError(f"'eos_token_id' must be an integer, got {eos!r}")
        return cls(vocab=read.integer("vocab"), width=read.integer("width"),
                   norm_eps=KeyReader(section(raw, "norm", "config.json")).number("eps"),
                   layers_json=json.dumps(layers, sort_keys=True), loop=read_loop(raw.get("loop"), len(layers)),
                   logit_softcap=None if raw.get("logit_softcap") is None else read.number("logit_softcap"), eos_token_id=eos)

    def to_dict(self) -> dict[str, Any]:
        data = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
                "layers": self.layers}
        if self.loop is not None:
            data["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        if self.logit_softcap is not None:
            data["logit_softcap"] = self.logit_softcap
        if self.eos_token_id is not None:
            data["eos_token_id"] = self.eos_token_id
        return data
