"""Small random Tugelorn models for the tests: configurations, their tensors."""
import numpy as np

from hybrid_models import write  # noqa: F401  (config.json and model.safetensors of a folder)
from ug_amd import rng


def window(heads, kv_heads, dim, vdim, size, rot, base=10000.0, factor=1.0, scale=None, mlp=None):
    return {"type": "attention", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5, "mask": {"size": size},
                                                       "rot": {"base": base, "dims": rot, "scaling": {"factor": factor}}}}


def full(heads, kv_heads, dim, vdim, coef, every, scale=None, mlp=None):
    return {"type": "attention_2", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5,
                                                         "q_temp": {"coef": coef, "every": every}}}


def delta(heads, kv_heads, dim, vdim, conv, mlp=None):
    return {"type": "channel_delta", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def ff(size, limit):
    return {"kind": "dense", "ff": size, "limit": limit}


def config(width, vocab, layers, mult, loop=None, eps=1e-5):
    c = {"architecture": "Tugelorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult, "layers": layers}
    return {**c, "loop": dict(zip(("start", "stop", "times"), loop))} if loop else c


# sizes that no tile divides, a delta rule in front, layers without a feed-forward, three passes over the middle
ODD = config(90, 101, [
    delta(6, 2, 18, 21, 3, ff(37, 1.5)),
    window(6, 3, 22, 27, 37, 14, base=500.0, factor=3.0, mlp=ff(75, 0.7)),
    full(4, 1, 17, 9, 0.7, 16),
    delta(3, 3, 35, 10, 5, ff(20, 3.0)),
    window(2, 2, 8, 13, 1, 8, base=77.0, scale=0.9),
], 0.4, (1, 4, 3), eps=3e-4)
# sizes the matrix kernels of a real model take (products with k >= 256); the embedding joins in front of layer 0
EVEN = config(256, 130, [
    window(4, 4, 128, 64, 64, 64, factor=1.5, mlp=ff(512, 1.0)),
    delta(4, 1, 64, 128, 4, ff(256, 2.5)),
    full(8, 2, 32, 128, 0.3, 40, mlp=ff(320, 1.2)),
    delta(2, 2, 128, 32, 2),
    window(6, 2, 64, 64, 100, 32),
], 0.7, (0, 2, 2))
# everything there can be one of
ONES = config(8, 3, [
    full(1, 1, 1, 1, 1.0, 1, mlp=ff(1, 1.0)),
    delta(1, 1, 1, 1, 1),
    window(1, 1, 2, 1, 1, 2, base=2.0, scale=1.0, mlp=ff(1, 0.5)),
    window(1, 1, 3, 2, 2, 0, base=2.0, scale=1.0),
], 1.0, (3, 4, 1))
MODELS = {"odd": ODD, "even": EVEN, "ones": ONES}
# (decay, output gate) ranks by layer; only the tensors say them
RANKS = {"odd": {0: (7, 5), 3: (12, 33)}, "even": {1: (16, 32), 3: (8, 24)}, "ones": {1: (1, 1)}}


def shapes(cfg, ranks):
    w, v, out = cfg["width"], cfg["vocab"], {}
    out["embed"] = (v, w)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        H, G, d, vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        out.update({p + "norm1": (w,), p + "norm1b": (w,)})
        if layer["type"] == "channel_delta":
            ra, rg = ranks[i]
            out.update({p + "mix.q": (G * d, w), p + "mix.k": (G * d, w), p + "mix.v": (H * vd, w), p + "mix.q.conv": (G * d, m["conv"]), p + "mix.k.conv": (G * d, m["conv"]),
                        p + "mix.v.conv": (H * vd, m["conv"]), p + "mix.b": (H, w), p + "mix.A_log": (H,), p + "mix.norm": (vd,), p + "mix.a1": (ra, w), p + "mix.a2": (H * d, ra),
                        p + "mix.dt_bias": (H * d,), p + "mix.g1": (rg, w), p + "mix.g2": (H * vd, rg)})
        else:
            out.update({p + "mix.q": (H * d, w), p + "mix.k": (G * d, w), p + "mix.v": (G * vd, w)})
            if layer["type"] == "attention_2":
                out.update({p + "mix.q.b": (H * d,), p + "mix.k.b": (G * d,), p + "mix.v.b": (G * vd,)})
        out[p + "mix.o"] = (w, H * vd)
        if layer["mlp"]:
            f = layer["mlp"]["ff"]
            out.update({p + "norm2": (w,), p + "norm2b": (w,), p + "mlp.gate": (f, w), p + "mlp.up": (f, w), p + "mlp.down": (w, f)})
    out["final.norm"], out["head"] = (w,), (v, w)
    return out


def weights(cfg, ranks, seed):
    """name -> float64 array of bf16 values.  Queries and keys are large enough for single keys to stand out, gates and ups for the
    feed-forward's limit to cut in, decays run from nearly nothing to nearly everything."""
    out = {}
    for i, (name, shape) in enumerate(shapes(cfg, ranks).items()):
        tail = name.split(".")[-1]
        x = rng.normal(seed * 1000 + i, int(np.prod(shape))).reshape(shape).astype(np.float64)
        if "norm" in tail:
            x = 1.0 + 0.2 * x
        elif tail == "A_log":
            x = 1.2 * x - 0.5
        elif tail == "dt_bias":
            x = 1.5 * x - 1.5
        elif tail == "conv":
            x = 0.6 * x
        elif len(shape) == 1:
            x = 0.5 * x
        elif tail in ("q", "k", "gate", "up"):
            x = x * (1.8 / np.sqrt(shape[-1]))
        elif name != "embed":
            x = x * (1.3 / np.sqrt(shape[-1]))
        out[name] = rng.bf16_round(x.astype(np.float32)).astype(np.float64)
    return out
