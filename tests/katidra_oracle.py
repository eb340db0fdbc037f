"""A plain float64 implementation of the Katidra design, written from its equations: whole sequences, no cache, no
batching, one function per mechanism.  It shares no code with the package; the tests compare the engine with it.

``tensors``: checkpoint name -> tensor; ``config``: the config.json dictionary.
"""

from __future__ import annotations

import math

import torch

F64 = torch.float64


def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def relu_squared(z):
    return torch.clamp(z, min=0.0) ** 2


# ----------------------------------------------------------------------------- linear attention with a fixed decay
def decayed_linear(q, k, v, decay):
    """q, k [T, H, D], v [T, H, V], decay [H]: S_t = decay S_(t-1) + k_t v_t^T, o_t = S_t^T q_t, S_(-1) = 0."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=F64)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = torch.einsum("hdv,hd->hv", S, q[t])
    return out


def decayed_linear_direct(q, k, v, decay):
    """The same as one sum over the earlier tokens: o_t = sum_(j <= t) decay^(t - j) (q_t . k_j) v_j."""
    T, H, _ = q.shape
    age = torch.arange(T, dtype=F64)[:, None] - torch.arange(T, dtype=F64)[None, :]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        w = torch.where(age >= 0, decay[h] ** age.clamp(min=0.0), torch.zeros(()).double())
        out[:, h] = (w * (q[:, h] @ k[:, h].T)) @ v[:, h]
    return out


def lightning(h, m, w, eps):
    T = h.shape[0]
    H, D, V = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    decay = torch.tensor([float(a) for a in m["decay"]], dtype=F64)
    q = silu(h @ w("q").T).view(T, H, D)
    k = silu(h @ w("k").T).view(T, H, D)
    v = silu(h @ w("v").T).view(T, H, V)
    y = decayed_linear(q, k, v, decay).reshape(T, H * V)
    y = rms_unit(y, eps) * w("norm") * torch.sigmoid(h @ w("g").T)       # all heads share one root mean square
    return y @ w("o").T


# ----------------------------------------------------------------------------- latent attention
def pair_frequencies(dims, base, scaling):
    """(radians per position of every pair, the factor on cos and sin)."""
    f, mag = [], 1.0
    for i in range(dims // 2):
        f.append(base ** (-2.0 * i / dims))
    if scaling:
        factor, original = float(scaling["factor"]), float(scaling["original"])
        where = lambda turns: dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
        lo = max(math.floor(where(float(scaling["fast"]))), 0)
        hi = min(math.ceil(where(float(scaling["slow"]))), dims - 1)
        for i in range(dims // 2):
            r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
            f[i] = f[i] / factor * r + f[i] * (1.0 - r)
        mag = 0.1 * math.log(factor) + 1.0
    return torch.tensor(f, dtype=F64), mag


def rotate_pairs(x, rot):
    """x [T, heads, dim]: the pairs (2i, 2i + 1) of the first ``dims`` dimensions turn with the position."""
    dims = int(rot["dims"])
    f, mag = pair_frequencies(dims, float(rot["base"]), rot.get("scaling"))
    ang = torch.arange(x.shape[0], dtype=F64)[:, None] * f[None, :]
    c, s = mag * torch.cos(ang)[:, None, :], mag * torch.sin(ang)[:, None, :]
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out = x.clone()
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def window_softmax(s, size):
    """Softmax over the rows of s [T, T]; row i sees columns i - size + 1 .. i (size 0: all up to i)."""
    T = s.shape[0]
    age = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    hide = (age < 0) | ((age >= size) if size else torch.zeros_like(age, dtype=torch.bool))
    return torch.softmax(s.masked_fill(hide, -math.inf), -1)


def latent_attention(h, m, w, eps):
    """Keys and values are up-projections of one normed low-rank row per token; one rotated key part is shared by the
    heads; queries come from a normed low-rank row as well; one sigmoid gate per head."""
    T = h.shape[0]
    H, D, R, V, C = int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"])
    cq = rms_unit(h @ w("dq").T, eps) * w("dq.norm")
    q = (cq @ w("uq").T).view(T, H, D + R)
    qn, qr = q[..., :D], rotate_pairs(q[..., D:], m["rot"])
    dkv = h @ w("dkv").T
    c = rms_unit(dkv[:, :C], eps) * w("dkv.norm")
    kr = rotate_pairs(dkv[:, C:].view(T, 1, R), m["rot"])[:, 0]
    kn = (c @ w("uk").T).view(T, H, D)
    v = (c @ w("uv").T).view(T, H, V)
    gate = torch.sigmoid(h @ w("g").T)                                   # [T, H]
    size = int((m.get("mask") or {}).get("size") or 0)
    out = torch.zeros(T, H, V, dtype=F64)
    for hd in range(H):
        s = (qn[:, hd] @ kn[:, hd].T + qr[:, hd] @ kr.T) * float(m["scale"])
        out[:, hd] = window_softmax(s, size) @ v[:, hd] * gate[:, hd:hd + 1]
    return out.reshape(T, H * V) @ w("o").T


MIXERS = {"lightning": lightning, "latent_attention": latent_attention}


# ----------------------------------------------------------------------------- model
def forward(tensors, config, tokens, after=None):
    """Logits [T, vocab] of one sequence; ``after`` (a list) receives the residual stream after every layer."""
    get = lambda name: tensors[name].to(F64)
    eps = float(config["norm"]["eps"])
    x = get("embed")[torch.as_tensor(tokens, dtype=torch.long)] * float(config["embedding"]["scale"])
    for i, L in enumerate(config["layers"]):
        j = L.get("weights_of")
        p = f"l{i if j is None else j}."
        w = lambda name, p=p: get(p + "mix." + name)
        y = MIXERS[L["type"]](x, L["mixer"], w, eps)
        x = x + rms_unit(y, eps) * get(p + "norm1")
        if L.get("mlp"):
            f = relu_squared(x @ get(p + "mlp.up").T) @ get(p + "mlp.down").T
            x = x + rms_unit(f, eps) * get(p + "norm2")
        if after is not None:
            after.append(x.clone())
    return (rms_unit(x, eps) * get("final.norm")) @ get("head").T


def greedy(tensors, config, prompt, n):
    """n tokens, each the arg-max of the last position's logits (lowest index on a tie)."""
    toks = list(prompt)
    out = []
    for _ in range(n):
        t = int(torch.argmax(forward(tensors, config, toks)[-1]))
        out.append(t)
        toks.append(t)
    return out
