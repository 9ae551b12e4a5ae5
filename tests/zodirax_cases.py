"""Small configurations and random weights of the Zodirax design, shared by its tests: every size differs from its neighbours unless a case
is about them being equal, weights are drawn so that every mechanism moves the logits, and are exact in bfloat16."""
import math

import torch


def scaling(factor=4.0, low=1.0, high=3.0, original=64):
    return {"factor": factor, "low": low, "high": high, "original": original}


def pair(heads=6, kv_heads=2, dim=40, vdim=24, rot_dims=28, base=700.0, scale=0.21, window=11, keep_first=3, stretch=scaling(), right_heads=3, right_dim=20,
         right_vdim=28, decay=None, left_scale=0.7, right_scale=1.3):
    rot = {"base": base, "dims": rot_dims}
    if stretch:
        rot["scaling"] = stretch
    decay = decay or [1 - 2.0 ** -(1 + 7 * i / max(1, right_heads - 1)) for i in range(right_heads)]
    return {"type": "parallel", "mixer": {
        "left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": window, "keep_first": keep_first}, "rot": rot},
        "right": {"heads": right_heads, "dim": right_dim, "vdim": right_vdim, "decay": decay}, "left_scale": left_scale, "right_scale": right_scale}}


def mamba(inner=90, state=5, dt_rank=7, conv=3):
    return {"type": "mamba1", "mixer": {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}}


def dense(ff=150):
    return {"kind": "dense", "ff": ff}


def config(layers, width=96, vocab=131, scale=0.75, eps=1e-5):
    return {"architecture": "Zodirax", "embedding": {"scale": scale}, "layers": [dict(mixer, mlp=mlp) for mixer, mlp in layers], "norm": {"eps": eps},
            "vocab": vocab, "width": width}


# name -> configuration
CASES = {
    # nothing is a multiple of anything, layers without a feed-forward, different windows
    "odd": config([(pair(), dense()), (mamba(), None), (mamba(inner=200, state=21, dt_rank=70, conv=5), dense(ff=40)),
                   (pair(heads=5, kv_heads=5, dim=24, vdim=20, rot_dims=24, window=50, keep_first=1, stretch=None, right_heads=2, right_dim=72, right_vdim=36), None)],
                  width=100),
    # sizes of ordinary layers
    "wide": config([(mamba(inner=256, state=16, dt_rank=20, conv=4), dense(ff=700)),
                    (pair(heads=8, kv_heads=2, dim=128, vdim=128, rot_dims=64, scale=0.08, window=33, keep_first=5, right_heads=2, right_dim=128, right_vdim=64),
                     dense(ff=256)),
                    (pair(heads=4, kv_heads=1, dim=72, vdim=64, rot_dims=72, window=200, keep_first=2, right_heads=1, right_dim=256, right_vdim=200), dense(ff=64))],
                   width=256, vocab=257),
    # larger than the register and matrix-core kernels take, more query heads per key head than a tile has rows
    "large_heads": config([(pair(heads=2, kv_heads=1, dim=200, vdim=136, rot_dims=100, scale=0.07, right_heads=1, right_dim=288, right_vdim=264), dense(ff=96)),
                           (pair(heads=20, kv_heads=1, dim=136, vdim=16, rot_dims=6, window=40, keep_first=70, right_heads=1), None),
                           (mamba(inner=64, state=100, dt_rank=130, conv=8), None)], width=128, vocab=64),
    # one of everything, nothing stretched, a window of one token, scales of one, a decay of exactly one
    "ones": config([(pair(heads=1, kv_heads=1, dim=32, vdim=32, rot_dims=32, window=1, keep_first=0, stretch=None, right_heads=1, right_dim=64, right_vdim=64, decay=[1.0],
                          left_scale=1.0, right_scale=1.0), dense(ff=64)), (mamba(inner=64, state=1, dt_rank=1, conv=1), dense(ff=16))], width=64, vocab=48, scale=1.0),
}


def tensor_shapes(cfg):
    """Names and shapes, written down independently of the product's own table."""
    W, V = cfg["width"], cfg["vocab"]
    s = {"embed": (V, W), "final.norm": (W,)}
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}.mix."
        s[f"l{i}.norm1"] = (W,)
        if layer["type"] == "mamba1":
            n, r, st = m["inner"], m["dt_rank"], m["state"]
            s |= {p + "in": (2 * n, W), p + "conv": (n, m["conv"]), p + "conv.b": (n,), p + "x": (r + 2 * st, n), p + "dt": (n, r), p + "dt.b": (n,),
                  p + "A_log": (n, st), p + "D": (n,), p + "o": (W, n)}
        else:
            a, r, pa, pr = m["left"], m["right"], p + "left.", p + "right."
            nq, nk, nv = a["heads"] * a["dim"], a["kv_heads"] * a["dim"], a["kv_heads"] * a["vdim"]
            s |= {pa + "q": (nq, W), pa + "k": (nk, W), pa + "v": (nv, W), pa + "q.b": (nq,), pa + "k.b": (nk,), pa + "v.b": (nv,), pa + "q.norm": (nq,),
                  pa + "k.norm": (nk,), pa + "sink": (a["heads"],), pa + "o": (W, a["heads"] * a["vdim"])}
            hq, hv = r["heads"] * r["dim"], r["heads"] * r["vdim"]
            s |= {pr + "q": (hq, W), pr + "k": (hq, W), pr + "v": (hv, W), pr + "g": (hv, W), pr + "o": (W, hv), pr + "norm": (hv,)}
        if layer["mlp"] is not None:
            n, p = layer["mlp"]["ff"], f"l{i}.mlp."
            s |= {f"l{i}.norm2": (W,), p + "gate": (n, W), p + "up": (n, W), p + "down": (W, n)}
    return s


def weights(cfg, seed=0):
    """{name: bfloat16 tensor}."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        t = torch.randn(*shape, generator=g)
        if name.endswith((".q.norm", ".k.norm", "right.norm", ".D")):
            t = 1 + 0.3 * t                               # (a skip well away from zero: without it all channels hang on the one sum B . C)
        elif "norm" in name:
            t = 0.3 * t                                   # stored around zero
        elif name == "embed":
            t = t / 2
        elif name.endswith("A_log"):
            t = 0.8 * t - 0.5
        elif name.endswith("dt.b"):
            t = 0.7 * t - 1.5
        elif name.endswith("conv"):
            t = t * (1.2 / math.sqrt(shape[-1]))
        elif len(shape) == 1:
            t = 0.7 * t                                   # biases, sinks
        else:
            t = t * (1.4 / math.sqrt(shape[-1]))
        out[name] = t.bfloat16()
    return out
