"""The Zisedra decoder as a ModelSpec: pre-norm blocks whose mixer is a recurrence by the gated delta rule ('delta') or
window attention beside such a recurrence with a decay a key channel ('side_by_side'), and whose feed-forward is a
mixture of experts with bounded gates beside a shared one, chosen by the sigmoids of a router's logits within the best
groups.  What a sublayer adds to the stream has a constant factor, which stands where each part can take it for
nothing (a norm's weights, the router's weights).  A run of layers may be gone through several times with the same
weights and a cache and state of its own each time; at the head of every pass the stream and the embedding output go
through a matrix together.  The embedding table is the output head too.

Tensor names: `embed`, `final.norm`, `loop.in`, and per layer i `l<i>.norm1`, `l<i>.norm2`,
`l<i>.mix.{q,k,v,o,b,a,g}`, `.mix.{q,k,v}.conv`, `.mix.{A_log,dt_bias,norm}`, or `l<i>.mix.left.{q,k,v,o}`,
`.mix.left.{q,k,v}.b`, `.mix.left.out`, `l<i>.mix.right.*` (with `a1`, `a2`, `g1`, `g2` for `a` and `g`) and
`.mix.right.out`, and `l<i>.mlp.{router,e<j>.{gate,up,down},shared.{gate,up,down}}` (no `.weight` suffix)."""
from __future__ import annotations

from ..config.zisedra_config import ZisedraAttention, ZisedraConfig, ZisedraDelta
from ..parts.rope import Rotary
from .model import LayerSpec, ModelSpec, ScheduleEntry


def zisedra_spec(cfg: ZisedraConfig) -> ModelSpec:
    W, eps, mult = cfg.width, cfg.norm_eps, cfg.residual_mult

    def norm(name: str):
        return ("rmsnorm", dict(name=name, width=W, eps=eps, suffix=""))

    def delta(m: ZisedraDelta, prefix: str, **more):
        return ("delta", dict(prefix=prefix, hidden=W, n_heads=m.heads, n_kv_heads=m.kv_heads, head_dim=m.dim, v_dim=m.vdim, conv_taps=m.conv,
                              eps=eps, decay_rank=m.decay_rank, gate_rank=m.gate_rank, **more))

    def attention(m: ZisedraAttention, prefix: str):
        position = None
        if m.rot_dims:
            scaling = None
            if m.scaling is not None:
                s = m.scaling
                scaling = dict(type="llama3", factor=s.factor, low_freq_factor=s.low, high_freq_factor=s.high,
                               original_max_position_embeddings=s.original)
            position = Rotary(m.dim, m.rot_dims, m.rot_base, pairing="interleaved", scaling=scaling)
        return ("attention", dict(prefix=prefix, hidden=W, n_heads=m.heads, n_kv_heads=m.kv_heads, head_dim=m.dim, v_dim=m.vdim, position=position,
                                  bias=True, scale=m.scale, window=m.window, eps=eps, names=("q", "k", "v", "o"), suffix="", bias_suffix=".b"))

    layers = []
    for i, L in enumerate(cfg.layers):
        p = f"l{i}."
        if L.type == "delta":
            mixer = delta(L.mixer, p + "mix.", gate="silu", out_scale=mult)
        else:
            mixer = ("side_by_side", dict(hidden=W, left=attention(L.left, p + "mix.left."), right=delta(L.right, p + "mix.right.", gate="sigmoid"),
                                          left_norm=p + "mix.left.out", right_norm=p + "mix.right.out", eps=eps, out_scale=mult))
        spec = LayerSpec(mixer=mixer, mixer_norm=norm(p + "norm1"), block="pre_norm")
        if L.second_norm:
            spec.ffn_norm = norm(p + "norm2")
        if L.mlp is not None:
            f = L.mlp
            spec.ffn = ("routed_moe", dict(prefix=p + "mlp.", hidden=W, n_experts=f.experts, top=f.top, intermediate=f.ff, groups=f.groups, keep=f.keep,
                                           group_score="best_two", correction=False, scores="sigmoid", renorm=False, limit=f.limit,
                                           shared_intermediate=f.shared_ff, shared_limit=f.shared_limit, out_scale=mult))
        layers.append(spec)
    schedule, parts = None, []
    if cfg.loop is not None:
        lp = cfg.loop
        parts.append(("part", "loop_entry", dict(matrix="loop.in", steps=None, width=W, times=lp.times)))
        schedule = [ScheduleEntry(i) for i in range(lp.start)]
        for t in range(lp.times):
            schedule += [ScheduleEntry(i, enter=(0, t) if i == lp.start else None) for i in range(lp.start, lp.stop)]
        schedule += [ScheduleEntry(i) for i in range(lp.stop, len(layers))]
    return ModelSpec(vocab_size=cfg.vocab, hidden_size=W, embed_name="embed", layers=layers, final_norm=norm("final.norm"), head_name="embed",
                     tie_head=True, schedule=schedule, stream_parts=parts)
