"""One registry from an architecture's name (config.json `architectures[0]`) to the
functions that read its configuration and describe its model.

The reference switches on the GGUF `general.architecture` string; llama, qwen2 and qwen3
all take its standard path and their optional features are found by tensor presence
(Daisi.Llogos.Cli/Program.cs:54-57, 101-103; Daisi.Llogos/Model/ModelLoader.cs:106-110).
Here each name states its defaults, and the loader checks them against the checkpoint."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Callable, Dict

from .model_config import ConfigError, DenseDecoderConfig


@dataclass(frozen=True)
class Architecture:
    name: str
    read_config: Callable[..., object]           # parsed config.json -> typed configuration
    model_spec: Callable[..., object]            # typed configuration (+ options) -> ModelSpec
    reads_shapes: bool = False                   # read_config also takes shapes={tensor name: shape} of the checkpoint,
                                                 # for sizes that the file leaves to the tensors


ARCHITECTURES: Dict[str, Architecture] = {}


def register_architecture(name: str, read_config: Callable[..., object],
                          model_spec: Callable[..., object], reads_shapes: bool = False) -> Architecture:
    arch = Architecture(name, read_config, model_spec, reads_shapes)
    ARCHITECTURES[name] = arch
    return arch


def architecture_of(data: dict) -> Architecture:
    archs = data.get("architectures") if isinstance(data, dict) else None
    if archs is None and isinstance(data, dict) and isinstance(data.get("architecture"), str):
        archs = [data["architecture"]]               # files that name one design in a string
    if not isinstance(archs, list) or not archs or not isinstance(archs[0], str):
        raise ConfigError("config.json: missing key 'architectures' (a list with the model's class name)")
    name = archs[0]
    if name not in ARCHITECTURES:
        raise ConfigError(f"unknown architecture '{name}'; known: {sorted(ARCHITECTURES)}")
    return ARCHITECTURES[name]


def _dense(name: str, bias_default: bool, qk_norm: bool) -> None:
    from ..models.dense_decoder import dense_decoder_spec

    def read(data: dict) -> DenseDecoderConfig:
        return DenseDecoderConfig.from_dict(data, attention_bias_default=bias_default, qk_norm=qk_norm)
    register_architecture(name, read, dense_decoder_spec)


_dense("LlamaForCausalLM", bias_default=False, qk_norm=False)
_dense("Qwen2ForCausalLM", bias_default=True, qk_norm=False)
_dense("Qwen3ForCausalLM", bias_default=False, qk_norm=True)


def _nipulorn() -> None:
    from ..models.nipulorn import nipulorn_spec
    from .nipulorn_config import NipulornConfig
    register_architecture("Nipulorn", NipulornConfig.from_dict, nipulorn_spec, reads_shapes=True)


_nipulorn()


def _zogurax() -> None:
    from ..models.zogurax import zogurax_spec
    from .zogurax_config import ZoguraxConfig
    register_architecture("Zogurax", ZoguraxConfig.from_dict, zogurax_spec)


_zogurax()


def _batodra() -> None:
    from ..models.batodra import batodra_spec
    from .batodra_config import BatodraConfig
    register_architecture("Batodra", BatodraConfig.from_dict, batodra_spec, reads_shapes=True)


_batodra()


def _zasidra() -> None:
    from ..models.zasidra import zasidra_spec
    from .zasidra_config import ZasidraConfig
    register_architecture("Zasidra", ZasidraConfig.from_dict, zasidra_spec)


_zasidra()


def _peponex() -> None:
    from ..models.peponex import peponex_spec
    from .peponex_config import PeponexConfig
    register_architecture("Peponex", PeponexConfig.from_dict, peponex_spec, reads_shapes=True)


_peponex()


def _zisedra() -> None:
    from ..models.zisedra import zisedra_spec
    from .zisedra_config import ZisedraConfig
    register_architecture("Zisedra", ZisedraConfig.from_dict, zisedra_spec, reads_shapes=True)


_zisedra()
