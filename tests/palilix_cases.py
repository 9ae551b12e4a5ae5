"""Small configurations and random weights of the Palilix design, shared by its tests: every size differs from its neighbours unless a
case is about them being equal, weights are drawn so that every mechanism moves the logits, and are exact in bfloat16."""
import copy
import math

import torch


def latent(heads=3, dim=24, rot_dim=8, vdim=40, kv_rank=56, scale=0.3, base=5000.0):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
                                                  "rot": {"base": base, "dims": rot_dim}}}


def retention(heads=5, dim=40, vdim=72, rot_dims=24, base=900.0, decay=None):
    decay = decay or [1 - 2.0 ** -(2 + 7 * i / max(1, heads - 1)) for i in range(heads)]
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay, "rot": {"base": base, "dims": rot_dims}}}


def dense(ff=150):
    return {"kind": "dense", "ff": ff}


def moe(experts=7, top=3, ff=40, limit=0.7, shared=None):
    out = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    if shared:
        out["shared"] = {"ff": shared[0], "limit": shared[1]}
    return out


def config(layers, width=96, vocab=131, loop=None, scale=3.0, logit_scale=1.5, softcap=12.0, eps=1e-5):
    cfg = {"architecture": "Palilix", "embedding": {"scale": scale}, "layers": [dict(mixer, mlp=mlp) for mixer, mlp in layers],
           "logit_scale": logit_scale, "logit_softcap": softcap, "norm": {"eps": eps}, "vocab": vocab, "width": width}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


# name -> configuration
CASES = {
    # nothing is a multiple of anything; a loop in the middle, three passes; every kind of feed-forward
    "odd": config([(latent(), moe(shared=(72, 0.9))), (retention(), dense()), (latent(heads=2, dim=40, rot_dim=24, vdim=24, kv_rank=72), None),
                   (retention(heads=3, dim=20, vdim=12, rot_dims=20), moe(experts=5, top=1, ff=24, limit=1.3))], width=100, loop=(1, 3, 3)),
    # sizes of ordinary layers, no loop
    "wide": config([(latent(heads=4, dim=128, rot_dim=64, vdim=128, kv_rank=512, scale=0.09), dense(ff=700)),
                    (retention(heads=2, dim=128, vdim=128, rot_dims=128), moe(experts=20, top=6, ff=64, limit=2.0, shared=(128, 1.0))),
                    (retention(heads=1, dim=256, vdim=200, rot_dims=64), dense(ff=64))], width=320, vocab=257),
    # larger than the register and matrix-core kernels take
    "large_heads": config([(latent(heads=1, dim=160, rot_dim=96, vdim=144, kv_rank=680, scale=0.07), dense(ff=96)),
                           (retention(heads=1, dim=288, vdim=264, rot_dims=288), None)], width=128, vocab=64, loop=(0, 2, 2)),
    # the whole stack looped, one head, every expert chosen, no softcap, a decay of exactly 1
    "ones": config([(latent(heads=1, dim=32, rot_dim=32, vdim=32, kv_rank=64, scale=0.15), moe(experts=4, top=4, ff=64, limit=0.5, shared=(64, 0.5))),
                    (retention(heads=3, dim=64, vdim=64, rot_dims=64, decay=[1.0, 0.25, 0.5]), moe(experts=1, top=1, ff=16, limit=1.0))],
                   width=64, vocab=48, loop=(0, 2, 2), softcap=None, scale=5.0, logit_scale=1.0),
}


def variant(name, **changes):
    cfg = copy.deepcopy(CASES[name])
    cfg.update(changes)
    return cfg


def tensor_shapes(cfg):
    """Names and shapes, written down independently of the product's own table."""
    W, V = cfg["width"], cfg["vocab"]
    s = {"embed": (V, W), "head": (V, W), "final.norm": (W,)}
    if cfg.get("loop"):
        s["loop.step"] = (cfg["loop"]["times"], W)
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}.mix."
        s[f"l{i}.norm1"] = (W,)
        H = m["heads"]
        if layer["type"] == "latent_attention":
            s |= {p + "q": (H * (m["dim"] + m["rot_dim"]), W), p + "dkv": (m["kv_rank"] + m["rot_dim"], W), p + "dkv.norm": (m["kv_rank"],),
                  p + "uk": (H * m["dim"], m["kv_rank"]), p + "uv": (H * m["vdim"], m["kv_rank"]), p + "o": (W, H * m["vdim"])}
        else:
            s |= {p + "q": (H * m["dim"], W), p + "k": (H * m["dim"], W), p + "v": (H * m["vdim"], W), p + "g": (H * m["vdim"], W),
                  p + "o": (W, H * m["vdim"])}
        f, p = layer["mlp"], f"l{i}.mlp."
        if f is None:
            continue
        if f["kind"] == "dense":
            s |= {p + "up": (f["ff"], W), p + "down": (W, f["ff"])}
        else:
            s[p + "router"] = (f["router"]["experts"], W)
            for e in range(f["router"]["experts"]):
                s |= {f"{p}e{e}.gate": (f["expert"]["ff"], W), f"{p}e{e}.up": (f["expert"]["ff"], W), f"{p}e{e}.down": (W, f["expert"]["ff"])}
            if f.get("shared"):
                n = f["shared"]["ff"]
                s |= {p + "shared.gate": (n, W), p + "shared.up": (n, W), p + "shared.down": (W, n)}
    return s


def weights(cfg, seed=0):
    """{name: bfloat16 tensor}."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        t = torch.randn(*shape, generator=g)
        if "norm" in name:
            t = 1 + 0.3 * t
        elif name == "embed":
            t = t / 2
        elif name == "loop.step":
            t = 0.7 * t
        elif name.endswith("router"):
            t = t * (6.0 / math.sqrt(shape[-1]))          # far apart: no close calls
        else:
            t = t * (1.4 / math.sqrt(shape[-1]))
        out[name] = t.bfloat16()
    return out
