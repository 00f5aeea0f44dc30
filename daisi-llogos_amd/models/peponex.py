"""The Peponex decoder as a ModelSpec: pre-norm blocks whose mixer is a recurrence with a matrix state and
a decay made from the token ('wkv'), a recurrence with a fixed decay a head ('lightning') or attention
through a latent over a sliding window ('latent_attention'), and whose feed-forward is SwiGLU or a mixture
of SwiGLU experts that a router weighs by its sigmoid scores, on the experts' inputs.  Behind its
feed-forward a layer takes its own part of a second embedding of the token into the stream.  A run of
layers may be gone through several times with the same weights and a cache and state of its own each time;
ahead of every pass the pass's own vector joins the stream, from the second pass on with the embedding
output.  The logits are bent through a tanh.

Tensor names: `embed`, `head`, `final.norm`, `side.embed`, `loop.step`, and per layer i `l<i>.norm1`,
`l<i>.norm2`, `l<i>.mix.*`, `l<i>.mlp.{gate,up,down}` or `l<i>.mlp.{router,e<j>.{gate,up,down}}`,
`l<i>.side.{gate,proj,norm}` (no `.weight` suffix)."""
from __future__ import annotations

from ..config.peponex_config import PeponexConfig
from ..parts.rope import Rotary
from .model import LayerSpec, ModelSpec, ScheduleEntry


def peponex_spec(cfg: PeponexConfig) -> ModelSpec:
    W, eps = cfg.width, cfg.norm_eps

    def norm(name: str):
        return ("rmsnorm", dict(name=name, width=W, eps=eps, suffix=""))

    layers = []
    for i, L in enumerate(cfg.layers):
        p, m = f"l{i}.", L.mixer
        common = dict(prefix=p + "mix.", hidden=W, n_heads=m.heads, eps=eps)
        if L.type == "wkv":
            mixer = ("wkv", dict(common, head_dim=m.dim, decay_rank=m.decay_rank))
        elif L.type == "lightning":
            mixer = ("lightning", dict(common, head_dim=m.dim, v_dim=m.vdim, decay=m.decay))
        else:
            position = Rotary(m.rot_dim, m.rot_dims, m.rot_base, pairing="split_half") if m.rot_dims else None
            mixer = ("latent_attention", dict(common, dim=m.dim, rot_dim=m.rot_dim, v_dim=m.vdim, q_rank=0, kv_rank=m.kv_rank,
                                              scale=m.scale, position=position, sink=False, window=m.window))
        spec = LayerSpec(mixer=mixer, mixer_norm=norm(p + "norm1"), block="pre_norm")
        if L.second_norm:
            spec.ffn_norm = norm(p + "norm2")
        if L.mlp is not None and L.mlp.kind == "dense":
            spec.ffn = ("swiglu", dict(prefix=p + "mlp.", hidden=W, intermediate=L.mlp.ff, names=("gate", "up", "down"), suffix=""))
        elif L.mlp is not None:
            spec.ffn = ("routed_moe", dict(prefix=p + "mlp.", hidden=W, n_experts=L.mlp.experts, top=L.mlp.top, intermediate=L.mlp.ff,
                                           correction=False, scores="sigmoid", renorm=False, weigh="input"))
        if cfg.side_dim:
            spec.more["tail"] = ("part", "token_side", dict(prefix=p + "side.", embedding="side.embed", hidden=W, vocab=cfg.vocab,
                                                            dim=cfg.side_dim, index=i, count=len(cfg.layers), eps=eps))
        layers.append(spec)
    schedule, parts = None, []
    if cfg.loop is not None:
        lp = cfg.loop
        parts.append(("part", "loop_add", dict(steps="loop.step", width=W, times=lp.times)))
        schedule = [ScheduleEntry(i) for i in range(lp.start)]
        for t in range(lp.times):
            schedule += [ScheduleEntry(i, enter=(0, t) if i == lp.start else None) for i in range(lp.start, lp.stop)]
        schedule += [ScheduleEntry(i) for i in range(lp.stop, len(layers))]
    return ModelSpec(vocab_size=cfg.vocab, hidden_size=W, embed_name="embed", layers=layers, final_norm=norm("final.norm"),
                     head_name="head", head_suffix="", schedule=schedule, stream_parts=parts, logit_softcap=cfg.logit_softcap)
