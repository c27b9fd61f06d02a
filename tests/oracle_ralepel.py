"""Plain float64 oracle of the Ralepel design: one function per mechanism,
whole sequences, no cache, no state carried between calls, no code shared
with the engine. `cfg` is the checkpoint's config.json as a dict, `W` maps
checkpoint tensor names to tensors.

Notation: T tokens, H query heads, G key/value heads, D query/key entries per
head (R of them rotated in latent attention), DV value entries per head, L
latent entries.
"""

from __future__ import annotations

import torch

F64 = torch.float64


def _w(W, name):
    return W[name].to(F64)


def lin(W, name, x):
    y = x @ _w(W, name).t()
    return y + _w(W, name + ".b") if name + ".b" in W else y


def unit_rms(x, eps):
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return unit_rms(x, eps) * w.to(F64)


def silu(z):
    return z * torch.sigmoid(z)


def slopes(H):
    """Distance penalty per position and head."""
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)],
                        dtype=F64)


def sink_softmax_mix(s, v, sink):
    """s [T, n] scores (-inf: unseen), v [n, DV], sink: one more score whose
    key has no value."""
    full = torch.cat([s, torch.full((s.shape[0], 1), float(sink),
                                    dtype=F64)], dim=1)
    return torch.softmax(full, -1)[:, :-1] @ v


def attention(W, pre, m, h, eps):
    """Windowed attention whose values are the projected keys before their
    norm, with a linear distance penalty and a learned sink."""
    T = h.shape[0]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    q = lin(W, pre + "q", h).view(T, H, D)
    v = lin(W, pre + "k", h).view(T, G, D)
    q, k = unit_rms(q, eps), unit_rms(v, eps)
    size = int((m.get("mask") or {}).get("size", 0))
    ages = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    seen = ages >= 0
    if size > 0:
        seen &= ages < size
    slope, sink = slopes(H), _w(W, pre + "sink")
    out = torch.zeros(T, H, D, dtype=F64)
    for hh in range(H):
        g = hh // (H // G)
        s = q[:, hh] @ k[:, g].t() * m["scale"] - slope[hh] * ages
        s = s.masked_fill(~seen, float("-inf"))
        out[:, hh] = sink_softmax_mix(s, v[:, g], sink[hh])
    return lin(W, pre + "o", out.reshape(T, H * D))


def turn_halves(x, rot):
    """x [T, ..., n]: entries i and i + dims/2 turn by
    position * base^(-2i/dims)."""
    dims = int(rot["dims"])
    half = dims // 2
    i = torch.arange(half, dtype=F64)
    f = torch.pow(torch.tensor(float(rot["base"]), dtype=F64),
                  -2.0 * i / dims)
    a = torch.arange(x.shape[0], dtype=F64)[:, None] * f
    a = a.view(x.shape[0], *([1] * (x.dim() - 2)), half)
    c, s = torch.cos(a), torch.sin(a)
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], dim=-1)


def latent_rows(W, pre, m, h, eps):
    """(latent [T, L], turned key part [T, R]) of a layer that has its own
    down-projection."""
    L = m["kv_rank"]
    down = lin(W, pre + "dkv", h)
    c = rms_norm(down[:, :L], W[pre + "dkv.norm"], eps)
    return c, turn_halves(down[:, L:], m["rot"])


def latent_attention(W, pre, m, h, rows):
    """rows: latent_rows of this layer, or of the layer it shares with."""
    T = h.shape[0]
    H, D, R, DV = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, kr = rows
    q = lin(W, pre + "q", h).view(T, H, D + R)
    qr = turn_halves(q[..., D:], m["rot"])
    k = lin(W, pre + "uk", c).view(T, H, D)
    v = lin(W, pre + "uv", c).view(T, H, DV)
    late = torch.arange(T)[None, :] > torch.arange(T)[:, None]
    out = torch.zeros(T, H, DV, dtype=F64)
    for hh in range(H):
        s = (q[:, hh, :D] @ k[:, hh].t() + qr[:, hh] @ kr.t()) * m["scale"]
        s = s.masked_fill(late, float("-inf"))
        out[:, hh] = torch.softmax(s, -1) @ v[:, hh]
    return lin(W, pre + "o", out.reshape(T, H * DV))


def gated_ff(W, pre, h):
    return lin(W, pre + "down",
               silu(lin(W, pre + "gate", h)) * lin(W, pre + "up", h))


def route(W, pre, m, h):
    """(weights [T, top], experts [T, top]): softmax over the largest
    biased logits."""
    z = lin(W, pre + "router", h)
    best, pick = torch.topk(z, int(m["router"]["top"]), dim=-1)
    return torch.softmax(best, -1), pick


def moe_ff(W, pre, m, h):
    out = torch.zeros_like(h)
    weights, pick = route(W, pre, m, h)
    for t in range(h.shape[0]):
        for w, e in zip(weights[t], pick[t].tolist()):
            out[t] += w * gated_ff(W, f"{pre}e{e}.", h[t])
    if m.get("shared"):
        out = out + torch.sigmoid(lin(W, pre + "shared.sg", h)) * gated_ff(
            W, pre + "shared.", h)
    return out


def feed_forward(W, pre, f, h):
    return gated_ff(W, pre, h) if f["kind"] == "dense" else moe_ff(
        W, pre, f, h)


def forward(cfg, W, tokens, streams=None):
    """tokens: list of ids of one sequence. Returns float64 logits
    [T, vocab]; `streams` (a list) receives the residual stream after every
    layer."""
    eps = cfg["norm"]["eps"]
    x = _w(W, "embed")[torch.as_tensor(tokens, dtype=torch.long)]
    cached = {}
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        if spec["type"] == "attention":
            y = attention(W, p + "mix.", m, x, eps)
        else:
            src = m.get("kv_from")
            if src is None:
                cached[i] = latent_rows(W, p + "mix.", m, x, eps)
                src = i
            y = latent_attention(W, p + "mix.", m, x, cached[src])
        x = x + rms_norm(y, W[p + "norm1"], eps)
        if spec.get("mlp") is not None:
            y = feed_forward(W, p + "mlp.", spec["mlp"], x)
            x = x + rms_norm(y, W[p + "norm2"], eps)
        if streams is not None:
            streams.append(x.clone())
    return rms_norm(x, W["final.norm"], eps) @ _w(W, "head").t()
