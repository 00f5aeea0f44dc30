"""Typed configuration of the Peponex decoder, read from its config.json.

The file names the design in `architecture`, gives `vocab`, `width`, `norm.eps`, optionally
`logit_softcap`, `token_side.dim` (the width of a layer's own part of the second embedding) and
`loop.{start, stop, times}` (layers start .. stop - 1 run `times` times in a row), and lists the
layers.  A layer entry has a `type`, the mixer's sizes and constants under `mixer`, and its
feed-forward under `mlp` (null: none).

    'wkv'               heads, dim (the decay's inner width is taken from the tensors, or from `decay_rank`)
    'lightning'         heads, dim, vdim, decay (a number a head)
    'latent_attention'  heads, dim, rot_dim, vdim, kv_rank, scale, rot.{base, dims}, mask.size (the window)

    mlp.kind 'dense'    ff
    mlp.kind 'moe'      expert.ff, router.{experts, top}

A layer without a feed-forward may still have the tensor of its second norm, which nothing reads: the
reader takes the tensors' shapes and looks for `l<i>.norm2`."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, Optional, Tuple

from .model_config import ConfigError, ConfigReader

LAYER_TYPES = ("wkv", "lightning", "latent_attention")


@dataclass(frozen=True)
class PeponexWkv:
    heads: int
    dim: int
    decay_rank: int


@dataclass(frozen=True)
class PeponexLightning:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]


@dataclass(frozen=True)
class PeponexLatent:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot_dims: int                # 0: nothing is rotated
    rot_base: float
    window: int                  # 0: every key up to the query's own


@dataclass(frozen=True)
class PeponexMlp:
    kind: str                    # 'dense' or 'moe'
    ff: int                      # dense: the width between the matrices; moe: an expert's
    experts: int = 0
    top: int = 0


@dataclass(frozen=True)
class PeponexLayer:
    type: str
    mixer: object                # PeponexWkv, PeponexLightning or PeponexLatent
    mlp: Optional[PeponexMlp]
    second_norm: bool            # the tensor l<i>.norm2 is there


@dataclass(frozen=True)
class PeponexLoop:
    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class PeponexConfig:
    architecture: str
    vocab: int
    width: int
    norm_eps: float
    logit_softcap: float         # 0: the logits as they are
    side_dim: int                # 0: no second embedding
    loop: Optional[PeponexLoop]
    layers: Tuple[PeponexLayer, ...]

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def eos_token_ids(self) -> Tuple[int, ...]:
        return ()

    @classmethod
    def from_dict(cls, data: dict, shapes: Optional[Dict[str, tuple]] = None) -> "PeponexConfig":
        r = ConfigReader(data)
        raw = r._raw("layers")
        if not isinstance(raw, list) or not raw:
            raise ConfigError("config.json: key 'layers' must be a list with at least one layer")
        width, vocab = r.int("width"), r.int("vocab")
        if vocab <= 0 or width <= 0:
            raise ConfigError("config.json: vocab and width must be positive")
        layers = []
        for i, entry in enumerate(raw):
            where = f"config.json layers[{i}]"
            lr = ConfigReader(entry, where)
            kind = lr.str("type")
            if kind not in LAYER_TYPES:
                raise ConfigError(f"{where}: unknown layer type '{kind}' ({', '.join(LAYER_TYPES)})")
            mr = ConfigReader(lr.obj("mixer"), where + ".mixer")
            if kind == "wkv":
                mixer = _wkv(mr, where, (shapes or {}).get(f"l{i}.mix.w1"), width)
            else:
                mixer = _lightning(mr, where) if kind == "lightning" else _latent(mr, where)
            mlp = lr.obj("mlp", None)
            mlp = _mlp(ConfigReader(mlp, where + ".mlp"), where) if mlp is not None else None
            layers.append(PeponexLayer(kind, mixer, mlp, mlp is not None or f"l{i}.norm2" in (shapes or {})))
        side = r.obj("token_side", None)
        side_dim = ConfigReader(side, "config.json token_side").int("dim") if side is not None else 0
        cap = r.float("logit_softcap", 0.0)
        if side_dim < 0 or cap < 0:
            raise ConfigError("config.json: token_side.dim and logit_softcap must not be negative")
        eps = ConfigReader(r.obj("norm"), "config.json norm").float("eps")
        return cls(r.str("architecture", "Peponex"), vocab, width, eps, cap, side_dim, _loop(r, len(layers)), tuple(layers))


def _loop(r: ConfigReader, n_layers: int) -> Optional[PeponexLoop]:
    lo = r.obj("loop", None)
    if lo is None:
        return None
    lr = ConfigReader(lo, "config.json loop")
    loop = PeponexLoop(lr.int("start"), lr.int("stop"), lr.int("times"))
    if not 0 <= loop.start < loop.stop <= n_layers or loop.times < 1:
        raise ConfigError(f"config.json loop: start {loop.start} and stop {loop.stop} must name layers of the {n_layers}, times be at least 1")
    return loop


def _wkv(mr: ConfigReader, where: str, w1_shape: Optional[tuple], width: int) -> PeponexWkv:
    rank = mr.int("decay_rank", None)
    if w1_shape is not None:
        rank = int(w1_shape[0])
    m = PeponexWkv(mr.int("heads"), mr.int("dim"), rank if rank is not None else max(16, width // 16))
    if min(m.heads, m.dim, m.decay_rank) <= 0:
        raise ConfigError(f"{where}.mixer: heads, dim and decay_rank must be positive")
    return m


def _lightning(mr: ConfigReader, where: str) -> PeponexLightning:
    dim = mr.int("dim")
    decay = mr._raw("decay")
    if not isinstance(decay, list) or any(isinstance(d, bool) or not isinstance(d, (int, float)) for d in decay):
        raise ConfigError(f"{where}.mixer: key 'decay' must be a list of numbers")
    m = PeponexLightning(mr.int("heads"), dim, mr.int("vdim", dim), tuple(float(d) for d in decay))
    if min(m.heads, m.dim, m.vdim) <= 0:
        raise ConfigError(f"{where}.mixer: heads, dim and vdim must be positive")
    if len(m.decay) != m.heads:
        raise ConfigError(f"{where}.mixer: decay has {len(m.decay)} numbers for {m.heads} heads")
    return m


def _latent(mr: ConfigReader, where: str) -> PeponexLatent:
    dim, rot_dim = mr.int("dim"), mr.int("rot_dim", 0)
    rot_dims, base = 0, 1.0
    ro = mr.obj("rot", None)
    if ro is not None:
        rr = ConfigReader(ro, where + ".mixer.rot")
        rot_dims, base = rr.int("dims", rot_dim), rr.float("base")
        if rot_dims < 0 or rot_dims % 2 or rot_dims > rot_dim or base <= 0:
            raise ConfigError(f"{where}.mixer.rot: dims must be even and within rot_dim, base positive")
    mask = mr.obj("mask", None)
    window = ConfigReader(mask, where + ".mixer.mask").int("size") if mask is not None else 0
    m = PeponexLatent(mr.int("heads"), dim, rot_dim, mr.int("vdim", dim), mr.int("kv_rank"), mr.float("scale"), rot_dims, base, window)
    if min(m.heads, m.dim, m.vdim, m.kv_rank) <= 0 or m.rot_dim < 0:
        raise ConfigError(f"{where}.mixer: heads, dim, vdim and kv_rank must be positive")
    if mask is not None and window < 1:
        raise ConfigError(f"{where}.mixer.mask: size must be at least 1")
    return m


def _mlp(fr: ConfigReader, where: str) -> PeponexMlp:
    kind = fr.str("kind", "dense")
    if kind == "dense":
        mlp = PeponexMlp("dense", fr.int("ff"))
    elif kind == "moe":
        rr = ConfigReader(fr.obj("router"), where + ".mlp.router")
        mlp = PeponexMlp("moe", ConfigReader(fr.obj("expert"), where + ".mlp.expert").int("ff"), rr.int("experts"), rr.int("top"))
        if not 1 <= mlp.top <= mlp.experts:
            raise ConfigError(f"{where}.mlp.router: top must lie within 1..experts")
    else:
        raise ConfigError(f"{where}.mlp: unknown feed-forward kind '{kind}' (dense, moe)")
    if mlp.ff <= 0:
        raise ConfigError(f"{where}.mlp: ff must be positive")
    return mlp
