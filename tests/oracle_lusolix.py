"""Plain float64 oracle of the Lusolix design: one function per mechanism,
whole sequences, no cache, no state carried between calls, no code shared
with the engine. `cfg` is the checkpoint's config.json as a dict, `W` maps
checkpoint tensor names to tensors.

Notation: T tokens, H heads, D unrotated / R rotated query and key entries
per head, DV value entries per head, L latent entries, K convolution taps.
"""

from __future__ import annotations

import torch

F64 = torch.float64


def _w(W, name):
    return W[name].to(F64)


def lin(W, name, x):
    return x @ _w(W, name).t()


def layer_norm(x, w, b, eps):
    mu = x.mean(-1, keepdim=True)
    var = (x - mu).pow(2).mean(-1, keepdim=True)
    return (x - mu) / torch.sqrt(var + eps) * w.to(F64) + b.to(F64)


def unit_rms(x, eps):
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def embed(W, ids):
    """Token row plus the row of its position."""
    return _w(W, "embed")[ids] + _w(W, "pos")[:len(ids)]


def input_conv(h, w):
    """h [T, C] -> h + conv(h); w [C, K], the last column weighs the current
    token, zeros before the start."""
    T, C = h.shape
    K = w.shape[1]
    ext = torch.cat([torch.zeros(K - 1, C, dtype=F64), h], dim=0)
    y = h.clone()
    for j in range(K):
        y = y + ext[j:j + T] * w.to(F64)[:, j]
    return y


def turn_pairs(x, rot):
    """x [T, ..., n]: neighbours (2i, 2i+1) of the first dims entries turn
    by position * base^(-2i/dims)."""
    dims = int(rot["dims"])
    i = torch.arange(dims // 2, dtype=F64)
    f = torch.pow(torch.tensor(float(rot["base"]), dtype=F64),
                  -2.0 * i / dims)
    a = torch.arange(x.shape[0], dtype=F64)[:, None] * f
    a = a.view(x.shape[0], *([1] * (x.dim() - 2)), dims // 2)
    c, s = torch.cos(a), torch.sin(a)
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    y = x.clone()
    y[..., 0:dims:2] = u * c - v * s
    y[..., 1:dims:2] = v * c + u * s
    return y


def latent_attention(W, pre, m, h, eps):
    T = h.shape[0]
    H, D, R = m["heads"], m["dim"], m["rot_dim"]
    DV, L = m.get("vdim", D), m["kv_rank"]
    cq = unit_rms(lin(W, pre + "dq", h), eps) * _w(W, pre + "dq.norm")
    q = lin(W, pre + "uq", cq).view(T, H, D + R)
    down = lin(W, pre + "dkv", h)
    c = unit_rms(down[:, :L], eps) * _w(W, pre + "dkv.norm")
    kr = turn_pairs(down[:, L:], m["rot"])                    # [T, R]
    qr = turn_pairs(q[..., D:], m["rot"])
    k = lin(W, pre + "uk", c).view(T, H, D)
    v = lin(W, pre + "uv", c).view(T, H, DV)
    size = int((m.get("mask") or {}).get("size", 0))
    gate = torch.sigmoid(lin(W, pre + "g", h))                # [T, H]
    ages = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    seen = ages >= 0
    if size > 0:
        seen &= ages < size
    out = torch.zeros(T, H, DV, dtype=F64)
    for hh in range(H):
        s = (q[:, hh, :D] @ k[:, hh].t() + qr[:, hh] @ kr.t()) * m["scale"]
        s = s.masked_fill(~seen, float("-inf"))
        out[:, hh] = (torch.softmax(s, -1) @ v[:, hh]) * gate[:, hh:hh + 1]
    return lin(W, pre + "o", out.reshape(T, H * DV))


def poly_norm(z, coef, eps):
    """a N(z) + b N(z^2) + c N(z^3) + e, N: divided by the root mean square
    of the row."""
    a, b, c, e = (float(v) for v in coef.to(F64))
    return (a * unit_rms(z, eps) + b * unit_rms(z * z, eps)
            + c * unit_rms(z * z * z, eps) + e)


def dense_ff(W, pre, h, eps):
    return lin(W, pre + "down", poly_norm(lin(W, pre + "up", h),
                                          W[pre + "act"], eps))


def table_ff(W, pre, m, h, ids):
    """Experts named by a table row per token id, plain mean of their
    outputs."""
    top = int(m["router"]["top"])
    out = torch.zeros_like(h)
    for t, tok in enumerate(ids.tolist()):
        for e in W[pre + "table"][tok].tolist():
            p = f"{pre}e{e}."
            y = silu(lin(W, p + "gate", h[t])) * lin(W, p + "up", h[t])
            out[t] += lin(W, p + "down", y) / top
    return out


def gate(W, name, h):
    return torch.sigmoid(lin(W, name, h) + _w(W, name + ".b"))


def layer(W, cfg, i, x, ids):
    spec = cfg["layers"][i]
    eps, m = cfg["norm"]["eps"], float(cfg["residual_mult"])
    pre = f"l{i}."
    if spec["type"] != "latent_attention":
        raise ValueError(spec["type"])
    h = layer_norm(x, W[pre + "norm1"], W[pre + "norm1.b"], eps)
    hc = input_conv(h, W[pre + "canon1"])
    y = latent_attention(W, pre + "mix.", spec["mixer"], hc, eps)
    x = x + m * (y * gate(W, pre + "rg1", h))
    f = spec.get("mlp")
    if f is not None:
        h = layer_norm(x, W[pre + "norm2"], W[pre + "norm2.b"], eps)
        if f["kind"] == "dense":
            y = dense_ff(W, pre + "mlp.", h, eps)
        else:
            y = table_ff(W, pre + "mlp.", f, h, ids)
        x = x + m * (y * gate(W, pre + "rg2", h))
    return x


def forward(cfg, W, tokens, streams=None):
    """tokens: list of ids of one sequence. Returns float64 logits
    [T, vocab]; `streams` (a list) receives the residual stream after every
    layer."""
    ids = torch.as_tensor(tokens, dtype=torch.long)
    x = embed(W, ids)
    for i in range(len(cfg["layers"])):
        x = layer(W, cfg, i, x, ids)
        if streams is not None:
            streams.append(x.clone())
    h = layer_norm(x, W["final.norm"], W["final.norm.b"],
                   cfg["norm"]["eps"])
    return h @ _w(W, "embed").t()
