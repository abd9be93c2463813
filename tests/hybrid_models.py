"""Small random Tanolorn models for the tests: configurations, their tensors, model folders."""
import json
import os

import numpy as np

from ug_amd import rng, st_writer


def latent(heads, dim, rot, vdim, q_rank, kv_rank, base=10000.0, scale=None, kv_from=None, mlp=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale or (dim + rot) ** -0.5,
         "rot": {"base": base, "dims": rot}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def ssm(heads, vdim, state, groups, norm_groups, conv, mlp=None):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "norm_groups": norm_groups, "conv": conv}, "mlp": mlp}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, count, keep):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "groups": {"count": count, "keep": keep}}}


def config(width, vocab, side, layers, eps=1e-5):
    return {"architecture": "Tanolorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "token_side": {"dim": side}, "layers": layers}


# sizes that no tile divides, a state-space layer in front, layers without a feed-forward, two layers on one cache
ODD = config(90, 101, 11, [
    ssm(6, 21, 19, 3, 2, 3, moe(37, 6, 2, 3, 2)),
    latent(3, 18, 14, 27, 35, 41, base=500.0),
    ssm(4, 10, 33, 1, 4, 5),
    latent(5, 22, 14, 9, 50, 41, base=500.0, kv_from=1, mlp=dense(75)),
    latent(2, 7, 6, 13, 20, 30, base=77.0, mlp=moe(21, 9, 4, 3, 2)),
], eps=3e-4)
# sizes the matrix kernels of a real model take (products with k >= 256, rotated parts apart from the rest)
EVEN = config(256, 130, 32, [
    latent(4, 64, 32, 48, 256, 128, mlp=dense(512)),
    ssm(8, 32, 64, 2, 4, 4, moe(256, 8, 3, 4, 2)),
    latent(2, 128, 64, 96, 64, 128, mlp=moe(320, 4, 2, 2, 1)),
    ssm(4, 64, 128, 4, 1, 4, dense(256)),
])
# everything there can be one of
ONES = config(8, 3, 1, [
    ssm(1, 1, 1, 1, 1, 1, moe(1, 1, 1, 1, 1)),
    latent(1, 1, 2, 1, 1, 1, base=2.0, scale=1.0, mlp=dense(1)),
    ssm(2, 3, 5, 2, 1, 1, moe(3, 2, 1, 2, 1)),
])


def shapes(cfg):
    w, v, side, out = cfg["width"], cfg["vocab"], cfg["token_side"]["dim"], {}
    out["embed"], out["side.embed"] = (v, w), (v, side * len(cfg["layers"]))
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        out[p + "norm1"] = (w,)
        if layer["type"] == "latent_attention":
            q = m["dim"] + m["rot_dim"]
            out.update({p + "mix.dq": (m["q_rank"], w), p + "mix.dq.norm": (m["q_rank"],), p + "mix.uq": (m["heads"] * q, m["q_rank"]),
                        p + "mix.uk": (m["heads"] * m["dim"], m["kv_rank"]), p + "mix.uv": (m["heads"] * m["vdim"], m["kv_rank"]),
                        p + "mix.o": (w, m["heads"] * m["vdim"])})
            if "kv_from" not in m:
                out.update({p + "mix.dkv": (m["kv_rank"] + m["rot_dim"], w), p + "mix.dkv.norm": (m["kv_rank"],)})
        else:
            inner, ch = m["heads"] * m["vdim"], m["heads"] * m["vdim"] + 2 * m["groups"] * m["state"]
            out.update({p + "mix.in": (inner + ch + m["heads"], w), p + "mix.conv": (ch, m["conv"]), p + "mix.conv.b": (ch,), p + "mix.dt_bias": (m["heads"],),
                        p + "mix.A_log": (m["heads"],), p + "mix.D": (m["heads"],), p + "mix.norm": (inner,), p + "mix.o": (w, inner)})
        f = layer["mlp"]
        if f:
            out[p + "norm2"] = (w,)
            if f["kind"] == "dense":
                out.update({p + "mlp.gate": (f["ff"], w), p + "mlp.gate.b": (f["ff"],), p + "mlp.up": (f["ff"], w), p + "mlp.up.b": (f["ff"],),
                            p + "mlp.down": (w, f["ff"]), p + "mlp.down.b": (w,)})
            else:
                n = f["router"]["experts"]
                out.update({p + "mlp.router": (n, w), p + "mlp.correction": (n,)})
                for e in range(n):
                    out.update({p + f"mlp.e{e}.gate": (f["expert"]["ff"], w), p + f"mlp.e{e}.up": (f["expert"]["ff"], w), p + f"mlp.e{e}.down": (w, f["expert"]["ff"])})
        out.update({p + "side.gate": (side, w), p + "side.proj": (w, side), p + "side.norm": (w,)})
    out["final.norm"], out["head"] = (w,), (v, w)
    return out


def weights(cfg, seed, steady_routing=False):
    """name -> float64 array of bf16 values.  steady_routing: choices of experts that rounding cannot turn (they hang on the
    correction more than on the row)."""
    out = {}
    for i, (name, shape) in enumerate(shapes(cfg).items()):
        n, tail = int(np.prod(shape)), name.split(".")[-1]
        x = rng.normal(seed * 1000 + i, n).reshape(shape).astype(np.float64)
        if tail in ("norm1", "norm2") or name == "final.norm":
            x = 0.1 * x                                            # stored around zero
        elif tail == "norm" or tail == "D":
            x = 1.0 + 0.2 * x
        elif tail == "A_log":
            x = 0.7 * x - 1.0
        elif tail == "dt_bias":
            x = x - 1.0
        elif tail == "correction":
            x = (1.5 if steady_routing else 0.3) * x - 0.6         # choice scores of either sign
        elif tail == "router":
            x = x * ((0.2 if steady_routing else 1.5) / np.sqrt(shape[-1]))
        elif len(shape) == 1:
            x = 0.3 * x
        elif name in ("embed", "side.embed"):
            pass
        else:
            x = x * (1.3 / np.sqrt(shape[-1]))
        out[name] = rng.bf16_round(x.astype(np.float32)).astype(np.float64)
    return out


def write(folder, cfg, w):
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    st_writer.write_safetensors(os.path.join(folder, "model.safetensors"),
                                [(k, "BF16", v.shape, rng.to_bf16_bits(v.astype(np.float32)).reshape(v.shape)) for k, v in w.items()])
    return str(folder)
