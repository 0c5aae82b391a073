"""Solulix as data: layers in the order config.json lists them, a stretch of them run several times.

The embedded row passes an RMS norm of its own.  A layer is x += mixer(n(x)) + ff(n(x)) with one plain RMS norm: the
`parallel` block.  Mixers: grouped-query attention without a rotation whose queries, keys and values pass short
convolutions over time, over a window beside the sequence's first positions, with one added to the softmax's denominator
(a sink of score 0); or a gated delta rule.  Feed-forward: SiLU-gated, or a mixture of squared-ReLU experts (softmax
scores, a correction for the choice, weights over their sum times a constant, identity experts) with a shared expert; or
none.  The layers of `loop` are scheduled once per pass with caches of their own; before a pass its vector, and before
every pass but the first the embedding's output, is added to the stream.
Tensor names: embed, embed.norm, loop.step, head, final.norm, l<i>.norm1,
l<i>.mix.{q,k,v}(.conv), .o; l<i>.mix.{q,k,v}(.conv), .{b,a,A_log,dt_bias,norm,g,o};
l<i>.mlp.{gate,up,down} or l<i>.mlp.router, .correction, l<i>.mlp.e<k>.{up,down}, l<i>.mlp.shared.{up,down}.
"""
from ..config.solulix import SolulixConfig
from ..registry import register_architecture
from .spec import LayerSpec, ModelSpec, ScheduleEntry


def _mixer(c, l):
    D, m = c.hidden_size, l.mixer
    if l.type == "attention":
        return ("attention", {"hidden_size": D, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim, "value_dim": m.vdim,
                              "query_scale": m.scale, "window": m.window, "keep_first": m.keep_first, "conv": m.conv, "sink": 0.0,
                              "position": ("none", {}), "precise_weights": True, "tensors": ("q", "k", "v", "o")})
    return ("gated_delta", {"hidden_size": D, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "key_dim": m.dim, "value_dim": m.vdim,
                            "conv_taps": m.conv, "norm_eps": c.norm_eps})


def _feed_forward(c, f):
    D = c.hidden_size
    if f is None:
        return None
    if f.kind == "dense":
        return ("gated_mlp", {"hidden_size": D, "intermediate_size": f.ff, "activation": "silu", "tensors": ("gate", "up", "down")})
    shared = None if f.shared_ff is None else (
        "plain_mlp", {"hidden_size": D, "intermediate_size": f.shared_ff, "activation": "relu2", "tensors": ("up", "down"), "prefix": "shared."})
    return ("routed_experts", {"hidden_size": D, "intermediate_size": f.ff, "n_experts": f.experts, "identity": f.identity, "top": f.top,
                               "limit": None, "expert_kind": "relu2", "tensors": ("up", "down"), "score": "softmax", "renormalize": True,
                               "correction": "correction", "weight_scale": f.router_scale, "shared": shared})


def _schedule(c):
    if c.loop is None:
        return [ScheduleEntry(i) for i in range(len(c.layers))]
    l = c.loop
    entries = [ScheduleEntry(i) for i in range(l.start)]
    for t in range(l.times):
        step = ("pass_step", {"size": c.hidden_size, "passes": l.times, "index": t, "origin": t > 0, "tensor": "step"})
        entries += [ScheduleEntry(i, before=step if i == l.start else None, before_prefix="loop.") for i in range(l.start, l.stop)]
    return entries + [ScheduleEntry(i) for i in range(l.stop, len(c.layers))]


def build_spec(c: SolulixConfig) -> ModelSpec:
    D = c.hidden_size
    norm = ("rms_norm", {"size": D, "eps": c.norm_eps, "tensor": "", "init": "gain"})
    layers = []
    for i, l in enumerate(c.layers):
        p = f"l{i}."
        ff = _feed_forward(c, l.mlp)
        prefixes = {"mixer": p + "mix.", "pre_norm": p + "norm1"}
        if ff is not None:
            prefixes["feed_forward"] = p + "mlp."
        layers.append(LayerSpec(block=("parallel", {}), mixer=_mixer(c, l), feed_forward=ff, norm=norm, prefixes=prefixes))
    return ModelSpec(
        architecture=c.architecture, hidden_size=D, vocab_size=c.vocab_size,
        embedding=("scaled_embedding", {"vocab_size": c.vocab_size, "hidden_size": D, "scale": 1.0, "tensor": "",
                                        "norm": ("rms_norm", {"size": D, "eps": c.norm_eps, "tensor": ".norm", "init": "gain"})}),
        embedding_prefix="embed", layers=layers, schedule=_schedule(c),
        final_norm=norm, final_norm_prefix="final.norm",
        head=("linear_head", {"vocab_size": c.vocab_size, "hidden_size": D, "softcap": None, "tensor": ""}),
        head_prefix="head", stop_ids=())


register_architecture(SolulixConfig.architecture, SolulixConfig, build_spec)
