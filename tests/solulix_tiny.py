"""The tests' own small Solulix configurations.

P mixes everything: attention layers with values larger and smaller than keys, windows shorter than a cache page and no
multiple of one, kept first positions fewer and more than a page, several and single kv heads, two, four and five taps;
delta layers with several heads per kv head and values of another size than keys; dense layers, mixtures with and
without identity and shared experts, a layer without a feed-forward; a loop over inner layers, run three times.
Q takes the values that hide faults when they are 1 or equal: one head everywhere, equal key and value sizes, one tap, no
kept positions, a window of one, one expert of which one is chosen, every router output chosen, a loop of one pass over
one layer, a width that no matrix-core kernel takes.
R has a window as long as the tests' sequences, no kept positions and no loop.
S is P's shape with the attentions' scores scaled up until a softmax picks single keys: a key that is lost, a window's
edge one place off or a kept position too many or too few then changes the logits by far more than any tolerance.
"""
import json
import os

from trapetum_amd.config import SolulixConfig
from trapetum_amd.weights import write_model_folder


def att(heads, kv, dim, vdim, conv, scale, size, keep):
    return {"conv": conv, "dim": dim, "heads": heads, "kv_heads": kv, "mask": {"keep_first": keep, "size": size}, "scale": scale, "vdim": vdim}


def delta(heads, kv, dim, vdim, conv):
    return {"conv": conv, "dim": dim, "heads": heads, "kv_heads": kv, "vdim": vdim}


def dense(ff):
    return {"ff": ff, "kind": "dense"}


def moe(ff, experts, identity, top, scale, shared=None):
    d = {"expert": {"ff": ff}, "kind": "moe", "router": {"experts": experts, "identity": identity, "scale": scale, "top": top}}
    if shared is not None:
        d["shared"] = {"ff": shared}
    return d


def layer(kind, mixer, mlp):
    return {"mixer": mixer, "mlp": mlp, "type": kind}


def config(layers, vocab, width, eps, loop=None):
    d = {"architecture": "Solulix", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width}
    if loop is not None:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    return d


def config_p(scale=1.0):
    return config([layer("attention", att(4, 2, 16, 24, 4, 0.3 * scale, 11, 5), dense(72)),
                   layer("delta", delta(6, 2, 24, 20, 2), moe(40, 5, 2, 3, 1.3, shared=24)),
                   layer("attention", att(3, 1, 24, 8, 2, 0.25 * scale, 20, 19), moe(33, 3, 0, 2, 0.8)),
                   layer("delta", delta(2, 1, 32, 48, 5), None),
                   layer("attention", att(6, 3, 32, 32, 3, 0.2 * scale, 34, 1), dense(50))],
                  211, 96, 1e-5, loop=(1, 4, 3))


def config_q():
    return config([layer("attention", att(1, 1, 12, 12, 1, 0.3, 1, 0), moe(20, 1, 0, 1, 1.0)),
                   layer("delta", delta(1, 1, 10, 10, 1), dense(30)),
                   layer("attention", att(2, 2, 10, 10, 2, 0.3, 1, 3), moe(18, 2, 1, 3, 1.0, shared=18))],
                  97, 50, 1e-6, loop=(0, 1, 1))


def config_r():
    return config([layer("delta", delta(4, 4, 16, 16, 4), dense(48)),
                   layer("attention", att(4, 4, 16, 16, 3, 0.25, 1000, 0), moe(24, 4, 4, 2, 2.0, shared=40))], 150, 64, 1e-3)


CONFIGS = {"P": (config_p(), dict(seed=51, sigma=0.12, sigma_norm=0.3)),
           "Q": (config_q(), dict(seed=52, sigma=0.15, sigma_norm=0.2)),
           "R": (config_r(), dict(seed=53, sigma=0.12, sigma_norm=0.3)),
           "S": (config_p(scale=10.0), dict(seed=54, sigma=0.12, sigma_norm=0.3))}


def make_folder(tmp_path, which):
    cfg, init = CONFIGS[which]
    folder = os.path.join(str(tmp_path), f"solulix_{which}")
    write_model_folder(SolulixConfig.from_dict(cfg), folder, **init)
    with open(os.path.join(folder, "config.json")) as f:
        assert json.load(f) == cfg                     # the configuration writes back what it read
    return folder


def draw(rng):
    """A configuration drawn at random: sizes, head counts, windows, kept positions, taps, constants, the order of layers and
    the loop."""
    def attention():
        kv = rng.choice([1, 2, 3])
        dim = rng.choice([8, 12, 16, 20, 32, 48])
        return att(kv * rng.choice([1, 2, 3]), kv, dim, rng.choice([8, 12, 16, 24, 40, dim]), rng.choice([1, 2, 3, 4]), rng.choice([0.2, 0.35]),
                   rng.choice([1, 2, 7, 16, 23, 64]), rng.choice([0, 1, 4, 16, 17, 30]))

    def gated_delta():
        kv = rng.choice([1, 2, 3])
        return delta(kv * rng.choice([1, 2, 3]), kv, rng.choice([4, 8, 16, 20, 40, 64]), rng.choice([4, 6, 16, 24, 33, 64]), rng.choice([1, 2, 3, 4]))

    def mlp():
        kind = rng.choice(["none", "dense", "moe", "moe"])
        if kind == "none":
            return None
        if kind == "dense":
            return dense(rng.choice([16, 40, 72]))
        experts, identity = rng.choice([1, 2, 4, 7]), rng.choice([0, 1, 3])
        return moe(rng.choice([8, 24, 40]), experts, identity, rng.randint(1, min(experts + identity, 4)), rng.choice([0.5, 1.0, 1.7]),
                   rng.choice([None, 8, 32]))
    makers = {"attention": attention, "delta": gated_delta}
    layers = []
    for _ in range(rng.randint(2, 5)):
        kind = rng.choice(list(makers))
        layers.append(layer(kind, makers[kind](), mlp()))
    start = rng.randrange(len(layers))
    loop = rng.choice([None, (start, rng.randint(start + 1, len(layers)), rng.randint(1, 3)), (0, len(layers), 2)])
    return config(layers, rng.choice([64, 101, 300]), rng.choice([24, 40, 64, 100]), rng.choice([1e-6, 1e-5]), loop=loop)
