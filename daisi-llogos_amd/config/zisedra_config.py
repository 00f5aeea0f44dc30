"""Typed configuration of the Zisedra decoder, read from its config.json.

The file names the design in `architecture`, gives `vocab`, `width`, `norm.eps`, optionally `residual_mult` (the factor
on what a sublayer adds to the stream) and `loop.{start, stop, times}` (layers start .. stop - 1 run `times` times in
a row), and lists the layers.  A layer entry has a `type`, the mixer's sizes and constants under `mixer`, and its
feed-forward under `mlp` (null: none).

    'delta'      heads, kv_heads, dim, vdim, conv (taps)
    'parallel'   left: heads, kv_heads, dim, vdim, scale, mask.size (the window), rot.{base, dims,
                 scaling.{factor, low, high, original}};  right: as 'delta'

    mlp.kind 'moe'      expert.{ff, limit}, router.{experts, top, groups.{count, keep}}, shared.{ff, limit}

The inner widths of the right mixer's decay and gate are taken from the tensors `l<i>.mix.right.a1` and `.g1`, or from
`decay_rank` and `gate_rank`.  A layer without a feed-forward may still have the tensor of its second norm, which
nothing reads: the reader takes the tensors' shapes and looks for `l<i>.norm2`."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, Optional, Tuple

from .model_config import ConfigError, ConfigReader

LAYER_TYPES = ("delta", "parallel")


@dataclass(frozen=True)
class ZisedraDelta:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    decay_rank: int = 0          # 0: one decay a head
    gate_rank: int = 0           # 0: the gate has one matrix


@dataclass(frozen=True)
class ZisedraScaling:
    factor: float
    low: float
    high: float
    original: float


@dataclass(frozen=True)
class ZisedraAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int                  # 0: every key up to the query's own
    rot_dims: int                # 0: nothing is rotated
    rot_base: float
    scaling: Optional[ZisedraScaling]


@dataclass(frozen=True)
class ZisedraMlp:
    ff: int
    limit: float
    experts: int
    top: int
    groups: int
    keep: int
    shared_ff: int               # 0: no shared expert
    shared_limit: float


@dataclass(frozen=True)
class ZisedraLayer:
    type: str
    mixer: Optional[ZisedraDelta]            # 'delta'
    left: Optional[ZisedraAttention]         # 'parallel'
    right: Optional[ZisedraDelta]
    mlp: Optional[ZisedraMlp]
    second_norm: bool                        # the tensor l<i>.norm2 is there


@dataclass(frozen=True)
class ZisedraLoop:
    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class ZisedraConfig:
    architecture: str
    vocab: int
    width: int
    norm_eps: float
    residual_mult: float
    loop: Optional[ZisedraLoop]
    layers: Tuple[ZisedraLayer, ...]

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def eos_token_ids(self) -> Tuple[int, ...]:
        return ()

    @classmethod
    def from_dict(cls, data: dict, shapes: Optional[Dict[str, tuple]] = None) -> "ZisedraConfig":
        r = ConfigReader(data)
        shapes = shapes or {}
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
            mixer = left = right = None
            if kind == "delta":
                mixer = _delta(mr, where + ".mixer")
            else:
                left = _attention(ConfigReader(mr.obj("left"), where + ".mixer.left"), where + ".mixer.left")
                right = _delta(ConfigReader(mr.obj("right"), where + ".mixer.right"), where + ".mixer.right", width,
                               shapes.get(f"l{i}.mix.right.a1"), shapes.get(f"l{i}.mix.right.g1"))
            mlp = lr.obj("mlp", None)
            mlp = _mlp(ConfigReader(mlp, where + ".mlp"), where + ".mlp") if mlp is not None else None
            layers.append(ZisedraLayer(kind, mixer, left, right, mlp, mlp is not None or f"l{i}.norm2" in shapes))
        eps = ConfigReader(r.obj("norm"), "config.json norm").float("eps")
        return cls(r.str("architecture", "Zisedra"), vocab, width, eps, r.float("residual_mult", 1.0), _loop(r, len(layers)), tuple(layers))


def _loop(r: ConfigReader, n_layers: int) -> Optional[ZisedraLoop]:
    lo = r.obj("loop", None)
    if lo is None:
        return None
    lr = ConfigReader(lo, "config.json loop")
    loop = ZisedraLoop(lr.int("start"), lr.int("stop"), lr.int("times"))
    if not 0 <= loop.start < loop.stop <= n_layers or loop.times < 1:
        raise ConfigError(f"config.json loop: start {loop.start} and stop {loop.stop} must name layers of the {n_layers}, times be at least 1")
    return loop


def _heads(mr: ConfigReader, where: str) -> Tuple[int, int, int, int]:
    heads, dim = mr.int("heads"), mr.int("dim")
    kv, vdim = mr.int("kv_heads", heads), mr.int("vdim", dim)
    if min(heads, kv, dim, vdim) <= 0 or heads % kv:
        raise ConfigError(f"{where}: heads, kv_heads, dim and vdim must be positive, heads a multiple of kv_heads")
    return heads, kv, dim, vdim


def _delta(mr: ConfigReader, where: str, width: int = 0, a1: Optional[tuple] = None, g1: Optional[tuple] = None) -> ZisedraDelta:
    """width > 0: the form whose decay and gate are of low rank."""
    heads, kv, dim, vdim = _heads(mr, where)
    conv = mr.int("conv")
    if conv < 1:
        raise ConfigError(f"{where}: conv must be at least 1")
    ranks = (0, 0)
    if width:
        rank = max(8, width // 16)
        ranks = (int(a1[0]) if a1 else mr.int("decay_rank", rank), int(g1[0]) if g1 else mr.int("gate_rank", rank))
        if min(ranks) <= 0:
            raise ConfigError(f"{where}: decay_rank and gate_rank must be positive")
    return ZisedraDelta(heads, kv, dim, vdim, conv, *ranks)


def _attention(mr: ConfigReader, where: str) -> ZisedraAttention:
    heads, kv, dim, vdim = _heads(mr, where)
    rot_dims, base, scaling = 0, 1.0, None
    ro = mr.obj("rot", None)
    if ro is not None:
        rr = ConfigReader(ro, where + ".rot")
        rot_dims, base = rr.int("dims", dim), rr.float("base")
        if rot_dims < 0 or rot_dims % 2 or rot_dims > dim or base <= 0:
            raise ConfigError(f"{where}.rot: dims must be even and within dim, base positive")
        sc = rr.obj("scaling", None)
        if sc is not None:
            sr = ConfigReader(sc, where + ".rot.scaling")
            scaling = ZisedraScaling(sr.float("factor"), sr.float("low"), sr.float("high"), sr.float("original"))
            if scaling.factor <= 0 or not 0 < scaling.low < scaling.high or scaling.original <= 0:
                raise ConfigError(f"{where}.rot.scaling: factor and original must be positive, low below high")
    mask = mr.obj("mask", None)
    window = ConfigReader(mask, where + ".mask").int("size") if mask is not None else 0
    if mask is not None and window < 1:
        raise ConfigError(f"{where}.mask: size must be at least 1")
    return ZisedraAttention(heads, kv, dim, vdim, mr.float("scale"), window, rot_dims, base, scaling)


def _mlp(fr: ConfigReader, where: str) -> ZisedraMlp:
    kind = fr.str("kind", "moe")
    if kind != "moe":
        raise ConfigError(f"{where}: unknown feed-forward kind '{kind}' (moe)")
    er = ConfigReader(fr.obj("expert"), where + ".expert")
    rr = ConfigReader(fr.obj("router"), where + ".router")
    experts, top = rr.int("experts"), rr.int("top")
    groups, keep = 1, 1
    gr = rr.obj("groups", None)
    if gr is not None:
        g = ConfigReader(gr, where + ".router.groups")
        groups, keep = g.int("count"), g.int("keep")
        if groups < 1 or experts % groups or not 1 <= keep <= groups:
            raise ConfigError(f"{where}.router.groups: count must divide experts, keep lie within 1..count")
    if not 1 <= top <= experts // groups * keep:
        raise ConfigError(f"{where}.router: top must lie within 1..experts of the kept groups")
    shared_ff, shared_limit = 0, 0.0
    sh = fr.obj("shared", None)
    if sh is not None:
        sr = ConfigReader(sh, where + ".shared")
        shared_ff, shared_limit = sr.int("ff"), sr.float("limit")
        if shared_ff <= 0 or shared_limit < 0:
            raise ConfigError(f"{where}.shared: ff must be positive, limit not negative")
    mlp = ZisedraMlp(er.int("ff"), er.float("limit"), experts, top, groups, keep, shared_ff, shared_limit)
    if mlp.ff <= 0 or mlp.limit < 0:
        raise ConfigError(f"{where}.expert: ff must be positive, limit not negative")
    return mlp
