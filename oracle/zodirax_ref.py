"""Plain restatement of the Zodirax decoder (test infrastructure only): one function per mechanism, a Python loop wherever a loop is
the definition, no cache, no batching, no fusion.  Everything runs in the dtype of the weights it is given (float64 in the tests).

A model is (config dict, {tensor name: tensor}); a sequence is a list of token ids; every function works on one sequence [T, ...].

    x_0 = E[token] * s
    layer:   x <- x + N1(mixer(x)),  x <- x + N2(ff(x))          N(y) = y / rms(y) * (1 + w): the sublayer's output is normed
    logits = E N(x)
"""
import math

import torch


# ------------------------------------------------------------------------------------------------ norms, activations, rotation
def rms_norm(x, eps, weight):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


def layer_norm(x, stored, eps):
    """The layers' own norm: its weight is stored around zero."""
    return rms_norm(x, eps, 1 + stored)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def frequencies(rot):
    """Angle per position of every rotated pair; long wavelengths are stretched by `factor`, short ones kept, a ramp between."""
    out = []
    s = rot.get("scaling")
    for i in range(rot["dims"] // 2):
        f = float(rot["base"]) ** (-2.0 * i / rot["dims"])
        if s:
            wave = 2 * math.pi / f
            if wave > s["original"] / s["low"]:
                f = f / s["factor"]
            elif wave >= s["original"] / s["high"]:
                mix = (s["original"] / wave - s["low"]) / (s["high"] - s["low"])
                f = (1 - mix) * f / s["factor"] + mix * f
        out.append(f)
    return out


def rotate(x, pos, rot):
    """x [..., D] at integer positions `pos` (broadcast over the leading axes of x but the last): pair (i, i + dims/2) of the first
    `dims` entries turns by pos * frequency i, the other entries pass."""
    half = rot["dims"] // 2
    a = pos.to(x.dtype).unsqueeze(-1) * torch.tensor(frequencies(rot), dtype=torch.float64).to(x.dtype)
    c, s = a.cos(), a.sin()
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], dim=-1)


def visible(i, j, mask):
    """Does position i see position j: the last `size` tokens with itself, and the first `keep_first` of the sequence."""
    return j <= i and (i - j < mask["size"] or j < mask["keep_first"])


# ------------------------------------------------------------------------------------------------ mixers
def window_attention(h, w, cfg, eps, pos0=0):
    """h [T, width] -> [T, width]: grouped-query softmax attention over a window and the first tokens, a sink in the denominator."""
    T = h.shape[0]
    H, G, dk, dv = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    pos = torch.arange(pos0, pos0 + T)[:, None]
    q, k, v = (h @ w[n].T + w[n + ".b"] for n in ("q", "k", "v"))
    q = rotate(rms_norm(q, eps, w["q.norm"]).view(T, H, dk), pos, cfg["rot"])
    k = rotate(rms_norm(k, eps, w["k.norm"]).view(T, G, dk), pos, cfg["rot"])
    v = v.view(T, G, dv)
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for i in range(T):
        seen = [j for j in range(T) if visible(i, j, cfg["mask"])]
        for head in range(H):
            g = head // (H // G)
            s = (k[seen, g] @ q[i, head]) * cfg["scale"]
            top = max(s.max(), w["sink"][head])
            e = torch.exp(s - top)
            out[i, head] = (e @ v[seen, g]) / (e.sum() + torch.exp(w["sink"][head] - top))
    return out.reshape(T, H * dv) @ w["o"].T


def lightning(h, w, cfg, eps, state=None):
    """h [T, width] -> ([T, width], state [H, dim, vdim]).  S <- decay S + k v^T, o = S^T q, token by token; one norm over all heads."""
    T = h.shape[0]
    H, dk, dv = cfg["heads"], cfg["dim"], cfg["vdim"]
    q, k, v = silu(h @ w["q"].T).view(T, H, dk), silu(h @ w["k"].T).view(T, H, dk), silu(h @ w["v"].T).view(T, H, dv)
    decay = torch.tensor(cfg["decay"], dtype=h.dtype)[:, None, None]
    S = torch.zeros(H, dk, dv, dtype=h.dtype) if state is None else state
    o = torch.zeros(T, H, dv, dtype=h.dtype)
    for t in range(T):
        S = decay * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    o = rms_norm(o.reshape(T, H * dv), eps, w["norm"])
    return (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T, S


def parallel(h, w, cfg, eps):
    left = window_attention(h, sub(w, "left."), cfg["left"], eps)
    right = lightning(h, sub(w, "right."), cfg["right"], eps)[0]
    return cfg["left_scale"] * left + cfg["right_scale"] * right


def causal_conv(x, w, b):
    """x [T, C], w [C, taps]: y_t = b + sum_i w_i x_(t - taps + 1 + i), nothing before the start."""
    T, taps = x.shape[0], w.shape[1]
    y = torch.zeros_like(x)
    for t in range(T):
        for i in range(taps):
            if t - taps + 1 + i >= 0:
                y[t] += w[:, i] * x[t - taps + 1 + i]
        y[t] += b
    return y


def selective_scan(x, dt, A, B, C, D, state=None):
    """x, dt [T, inner], A [inner, N], B, C [T, N] -> (y [T, inner], state [inner, N])."""
    S = torch.zeros_like(A) if state is None else state
    y = torch.zeros_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + D * x[t]
    return y, S


def mamba(h, w, cfg):
    inner, r, n = cfg["inner"], cfg["dt_rank"], cfg["state"]
    x, z = (h @ w["in"].T).split([inner, inner], dim=-1)
    x = silu(causal_conv(x, w["conv"], w["conv.b"]))
    dt, B, C = (x @ w["x"].T).split([r, n, n], dim=-1)
    dt = softplus(dt @ w["dt"].T + w["dt.b"])
    y, _ = selective_scan(x, dt, -torch.exp(w["A_log"]), B, C, w["D"])
    return (y * silu(z)) @ w["o"].T


# ------------------------------------------------------------------------------------------------ feed-forward
def dense_ff(h, w):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


# ------------------------------------------------------------------------------------------------ the model
def sub(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens, taps=None):
    """Logits [T, vocab] of one sequence; `taps`, a list, receives the residual stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = weights["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    for i, lc in enumerate(cfg["layers"]):
        mix = sub(weights, f"l{i}.mix.")
        y = parallel(x, mix, lc["mixer"], eps) if lc["type"] == "parallel" else mamba(x, mix, lc["mixer"])
        x = x + layer_norm(y, weights[f"l{i}.norm1"], eps)
        if lc["mlp"]:
            x = x + layer_norm(dense_ff(x, sub(weights, f"l{i}.mlp.")), weights[f"l{i}.norm2"], eps)
        if taps is not None:
            taps.append(x)
    return layer_norm(x, weights["final.norm"], eps) @ weights["embed"].T
