"""The tests' own small Kaderax configurations.

P mixes everything: latent-attention layers whose rotation covers the rotated part, parallel layers with values larger and
smaller than keys, single and several kv heads, bias tables that reach to distances inside and beyond the tests' sequences,
temperatures that change every few positions, decays from almost none to almost all; a layer without a feed-forward; a loop
over inner layers, run three times.
Q takes the values that hide faults when they are 1 or equal: one head everywhere, equal sizes, one residual, scales of one, a
temperature that changes at every position, a bias table of two rows, a decay of one and a decay of zero, a loop of one pass,
sizes that no matrix-core kernel takes.
R starts its loop at the first layer and ends it at the last, twice; T has no loop.
S is P's shape with scores so sharp that a softmax picks single keys: a lost key or a bias one place off then changes the
logits by far more than any tolerance.
"""
import json
import os

from trapetum_amd.config import KaderaxConfig
from trapetum_amd.weights import write_model_folder


def latent(heads, dim, rot_dim, vdim, kv_rank, q_rank, scale, base=10000.0, dims=None):
    return {"dim": dim, "heads": heads, "kv_rank": kv_rank, "q_rank": q_rank, "rot": {"base": base, "dims": rot_dim if dims is None else dims},
            "rot_dim": rot_dim, "scale": scale, "vdim": vdim}


def left(heads, kv, dim, vdim, scale, softcap, bias_max, coef, every):
    return {"bias_max": bias_max, "dim": dim, "heads": heads, "kv_heads": kv, "q_temp": {"coef": coef, "every": every}, "scale": scale,
            "softcap": softcap, "vdim": vdim}


def right(dim, vdim, *decay):
    return {"decay": list(decay), "dim": dim, "heads": len(decay), "vdim": vdim}


def par(l, ls, r, rs):
    return {"left": l, "left_scale": ls, "right": r, "right_scale": rs}


def layer(mixer, ff):
    kind = "parallel" if "left" in mixer else "latent_attention"
    return {"mixer": mixer, "mlp": None if ff is None else {"ff": ff, "kind": "dense"}, "type": kind}


def config(layers, vocab, width, eps, mult, loop=None):
    d = {"architecture": "Kaderax", "layers": layers, "norm": {"eps": eps}, "residual_mult": mult, "vocab": vocab, "width": width}
    if loop is not None:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    return d


def config_p(sharp=1.0):
    return config([layer(latent(4, 16, 8, 24, 24, 20, 0.3 * sharp), 72),
                   layer(par(left(4, 2, 16, 24, 0.3 * sharp, 15.0 * sharp, 40, 0.4, 7), 0.7, right(24, 20, 0.6, 0.95, 0.999), 0.6), 40),
                   layer(latent(3, 8, 16, 12, 32, 28, 0.25 * sharp, base=500.0), None),
                   layer(par(left(3, 1, 24, 8, 0.25 * sharp, 8.0 * sharp, 200, -0.1, 16), 0.5, right(32, 48, 0.9, 0.3), 0.8), 64),
                   layer(latent(6, 32, 16, 32, 48, 40, 0.2 * sharp), 50)],
                  211, 96, 1e-5, 0.4, loop=(1, 4, 3))


def config_q():
    return config([layer(par(left(1, 1, 10, 10, 0.3, 5.0, 3, 1.0, 1), 1.0, right(10, 10, 1.0), 1.0), 30),
                   layer(latent(1, 10, 2, 10, 10, 10, 0.3), 20),
                   layer(par(left(2, 2, 10, 10, 0.3, 30.0, 17, 0.3, 1000), 1.0, right(6, 14, 0.0, 0.5), 1.0), None)],
                  97, 50, 1e-6, 1.0, loop=(1, 2, 1))


def config_r():
    return config([layer(latent(4, 16, 8, 16, 24, 24, 0.25), 48),
                   layer(par(left(4, 4, 16, 16, 0.25, 20.0, 64, 0.5, 32), 0.6, right(16, 16, 0.7, 0.8, 0.9, 0.99), 0.5), 56)],
                  150, 64, 1e-3, 0.5, loop=(0, 2, 2))


def config_t():
    return config([layer(par(left(6, 2, 32, 32, 0.2, 10.0, 25, 0.2, 10), 0.9, right(40, 16, 0.97, 0.85), 1.1), 40),
                   layer(latent(2, 24, 8, 16, 40, 16, 0.2), 33)], 130, 72, 1e-5, 0.7)


CONFIGS = {"P": (config_p(), dict(seed=61, sigma=0.12, sigma_norm=0.3)),
           "Q": (config_q(), dict(seed=62, sigma=0.15, sigma_norm=0.2)),
           "R": (config_r(), dict(seed=63, sigma=0.12, sigma_norm=0.3)),
           "T": (config_t(), dict(seed=65, sigma=0.12, sigma_norm=0.3)),
           "S": (config_p(sharp=10.0), dict(seed=64, sigma=0.12, sigma_norm=0.3))}


def make_folder(tmp_path, which):
    cfg, init = CONFIGS[which]
    folder = os.path.join(str(tmp_path), f"kaderax_{which}")
    write_model_folder(KaderaxConfig.from_dict(cfg), folder, **init)
    with open(os.path.join(folder, "config.json")) as f:
        assert json.load(f) == cfg                     # the configuration writes back what it read
    return folder


def draw(rng):
    """A configuration drawn at random: sizes, head counts, constants, the order of layers and the loop."""
    def latent_attention():
        rot = rng.choice([2, 4, 8, 16, 32])
        return latent(rng.choice([1, 2, 3, 4, 6]), rng.choice([8, 12, 16, 40]), rot, rng.choice([8, 12, 24, 40]),
                      rng.choice([8, 16, 24, 32, 48, 56]), rng.choice([8, 20, 32]), rng.choice([0.2, 0.35]), base=rng.choice([100.0, 500000.0]))

    def parallel():
        kv, n = rng.choice([1, 2, 3]), rng.choice([1, 2, 3, 5])
        dim = rng.choice([8, 12, 16, 20, 32, 48])
        return par(left(kv * rng.choice([1, 2, 3]), kv, dim, rng.choice([8, 12, 16, 24, 40, dim]), rng.choice([0.2, 0.35]), rng.choice([4.0, 20.0]),
                        rng.choice([17, 33, 50, 300]), rng.choice([0.1, 0.5]), rng.choice([1, 5, 16, 64])), rng.choice([0.5, 1.0]),
                   right(rng.choice([4, 8, 16, 20, 40, 64]), rng.choice([4, 6, 16, 24, 33, 64]), *[rng.choice([0.2, 0.7, 0.95, 0.9995]) for _ in range(n)]),
                   rng.choice([0.4, 1.0]))
    layers = []
    for _ in range(rng.randint(2, 5)):
        layers.append(layer(rng.choice([latent_attention, parallel])(), rng.choice([None, 16, 40, 72])))
    start = rng.randrange(len(layers))
    loop = rng.choice([None, (start, rng.randint(start + 1, len(layers)), rng.randint(1, 3)), (0, len(layers), 2)])
    return config(layers, rng.choice([64, 101, 300]), rng.choice([24, 40, 64, 100]), rng.choice([1e-6, 1e-5]), rng.choice([0.3, 1.0]), loop=loop)
