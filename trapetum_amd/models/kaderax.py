"""Kaderax as data: layers in the order config.json lists them, a stretch of them run several times.

A layer is x += m mixer(n1(x)), x += m ff(n2(x)) with plain RMS norms and a constant m of the model: the `pre_norm` block with
a residual scale.  Mixers: attention through a cached latent with a latent for the queries too, a rotation of neighbouring
pairs, a sink per head and a sigmoid gate per element; or `parallel`: grouped-query attention without a rotation (a
temperature of the query's position, a score cap, a learned bias per distance and head, a gate per head) beside linear
attention with a constant decay per head, added with a constant each.  Feed-forward: gelu-gated, or none.  The layers of
`loop` are scheduled once per pass with caches of their own; before every pass the stream becomes W [stream; embedding].
Tensor names: embed, loop.in, head, final.norm, l<i>.norm1/.norm2, l<i>.mix.{dq,dq.norm,uq,dkv,dkv.norm,uk,uv,sink,g,o};
l<i>.mix.left.{q,k,v,rel,g,o}, l<i>.mix.right.{q,k,v,g,o,norm}; l<i>.mlp.{gate,up,down}.
"""
from ..config.kaderax import KaderaxConfig
from ..registry import register_architecture
from .spec import LayerSpec, ModelSpec, ScheduleEntry


def _mixer(c, l):
    D, m = c.hidden_size, l.mixer
    if l.type == "latent_attention":
        position = ("rope", {"rotary_dim": m.rot_dims, "theta": m.rot_base, "pairing": "neighbours"}) if m.rot_dims else ("none", {})
        return ("latent_attention", {"hidden_size": D, "num_heads": m.heads, "nope_dim": m.dim, "rope_dim": m.rot_dim,
                                     "value_dim": m.vdim, "latent_rank": m.kv_rank, "scale": m.scale, "latent_eps": c.norm_eps,
                                     "position": position, "query_rank": m.q_rank, "output_gate": "g", "gate_per": "element",
                                     "sink": "sink", "joint_input": True, "precise_weights": True})
    a, r = m.left, m.right
    left = ("attention", {"hidden_size": D, "num_heads": a.heads, "num_kv_heads": a.kv_heads, "head_dim": a.dim, "value_dim": a.vdim,
                          "query_scale": a.scale, "softcap": a.softcap, "position": ("none", {}), "output_gate": "head",
                          "query_temperature": (a.temp_coef, a.temp_every), "distance_bias": "rel", "bias_reach": a.bias_max,
                          "bias_rows": max(2, min(32, 2 * (a.bias_max // 2))), "precise_weights": True,
                          "tensors": ("q", "k", "v", "o", "g")})
    right = ("linear_attention", {"hidden_size": D, "num_heads": r.heads, "key_dim": r.dim, "value_dim": r.vdim, "decay": r.decay,
                                  "norm_eps": c.norm_eps})
    return ("parallel", {"hidden_size": D, "left": left, "right": right, "combine": "weighted_sum",
                         "weights": (m.left_scale, m.right_scale), "deferred": True})


def _schedule(c):
    if c.loop is None:
        return [ScheduleEntry(i) for i in range(len(c.layers))]
    l = c.loop
    mix = ("stream_mix", {"size": c.hidden_size, "tensor": "in"})
    entries = [ScheduleEntry(i) for i in range(l.start)]
    for _ in range(l.times):
        entries += [ScheduleEntry(i, before=mix if i == l.start else None, before_prefix="loop.") for i in range(l.start, l.stop)]
    return entries + [ScheduleEntry(i) for i in range(l.stop, len(c.layers))]


def build_spec(c: KaderaxConfig) -> ModelSpec:
    D = c.hidden_size
    norm = ("rms_norm", {"size": D, "eps": c.norm_eps, "tensor": "", "init": "gain"})
    layers = []
    for i, l in enumerate(c.layers):
        p = f"l{i}."
        ff = None if l.mlp is None else ("gated_mlp", {"hidden_size": D, "intermediate_size": l.mlp.ff, "activation": "gelu_tanh",
                                                       "tensors": ("gate", "up", "down")})
        prefixes = {"mixer": p + "mix.", "pre_mixer_norm": p + "norm1"}
        if ff is not None:
            prefixes.update({"feed_forward": p + "mlp.", "pre_ff_norm": p + "norm2"})
        layers.append(LayerSpec(block=("pre_norm", {"residual_scale": c.residual_mult}), mixer=_mixer(c, l), feed_forward=ff, norm=norm,
                                prefixes=prefixes))
    return ModelSpec(
        architecture=c.architecture, hidden_size=D, vocab_size=c.vocab_size,
        embedding=("scaled_embedding", {"vocab_size": c.vocab_size, "hidden_size": D, "scale": 1.0, "tensor": ""}),
        embedding_prefix="embed", layers=layers, schedule=_schedule(c),
        final_norm=norm, final_norm_prefix="final.norm",
        head=("linear_head", {"vocab_size": c.vocab_size, "hidden_size": D, "softcap": None, "tensor": ""}),
        head_prefix="head", stop_ids=())


register_architecture(KaderaxConfig.architecture, KaderaxConfig, build_spec)
