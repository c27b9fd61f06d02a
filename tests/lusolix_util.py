"""Helpers for the Lusolix tests: small configurations in the checkpoint's
own config.json layout and random bf16 weights under the checkpoint's tensor
names. Checkpoint folders, engines and error measures come from
nanurax_util."""

from __future__ import annotations

import torch

from nanurax_util import (TOL, make_engine, rel_err,  # noqa: F401
                          row_errs, save_checkpoint)


def close(got, want, dtype):
    """Every row within 2e-4 in float32. In bfloat16 every row within 6e-2
    and the median row within 3e-2: nothing in this design turns a rounding
    error into a jump (the routing is a table)."""
    e = row_errs(got, want).sort().values
    ok = bool(e[-1] < TOL[dtype])
    if dtype != "float32":
        ok = ok and bool(e[len(e) // 2] < 3e-2)
    if not ok:
        print("row errors:", [round(float(x), 5) for x in e])
    return ok


def mixer(heads=3, dim=12, rot_dim=8, vdim=20, kv_rank=24, q_rank=32,
          size=20, scale=0.25, base=1000.0):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
         "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale,
         "rot": {"base": base, "dims": rot_dim}}
    if size:
        m["mask"] = {"size": size}
    return {"type": "latent_attention", "mixer": m}


def dense(ff=80):
    return {"kind": "dense", "ff": ff}


def moe(ff=24, experts=5, top=2):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top}}


def make_cfg(layers, width=64, vocab=97, eps=1e-5, taps=3, mult=0.6,
             positions=512):
    """layers: [(mixer dict, mlp dict | None)]."""
    return {
        "architecture": "Lusolix", "vocab": vocab, "width": width,
        "max_positions": positions, "norm": {"eps": eps},
        "canon": {"taps": taps}, "residual_mult": mult,
        "layers": [dict(m, mlp=f) for m, f in layers],
    }


def make_weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    W = {}

    def lin(name, out, inp, gain=1.0):
        W[name] = (torch.randn(out, inp, generator=g) * gain
                   / inp ** 0.5).to(torch.bfloat16)

    def vec(name, n, mean=0.0, std=1.0):
        W[name] = (mean + std * torch.randn(n, generator=g)).to(
            torch.bfloat16)

    width, vocab = cfg["width"], cfg["vocab"]
    taps = cfg["canon"]["taps"]
    lin("embed", vocab, width, width ** 0.5 * 0.4)
    lin("pos", cfg["max_positions"], width, width ** 0.5 * 0.2)
    vec("final.norm", width, 1.0, 0.1)
    vec("final.norm.b", width, 0.0, 0.1)
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        vec(p + "norm1", width, 1.0, 0.15)
        vec(p + "norm1.b", width, 0.0, 0.15)
        W[p + "canon1"] = (0.4 * torch.randn(width, taps, generator=g)).to(
            torch.bfloat16)
        lin(p + "rg1", width, width, 1.5)
        vec(p + "rg1.b", width, 0.3, 0.5)
        m, mp = layer["mixer"], p + "mix."
        H, D, R = m["heads"], m["dim"], m["rot_dim"]
        DV, L, Q = m["vdim"], m["kv_rank"], m["q_rank"]
        lin(mp + "dq", Q, width)
        vec(mp + "dq.norm", Q, 1.0, 0.3)
        lin(mp + "uq", H * (D + R), Q, 1.7)
        lin(mp + "dkv", L + R, width)
        vec(mp + "dkv.norm", L, 1.0, 0.3)
        lin(mp + "uk", H * D, L, 1.7)
        lin(mp + "uv", H * DV, L)
        lin(mp + "g", H, width, 1.5)
        lin(mp + "o", width, H * DV, 1.5)
        f = layer.get("mlp")
        if f is None:
            continue
        vec(p + "norm2", width, 1.0, 0.15)
        vec(p + "norm2.b", width, 0.0, 0.15)
        lin(p + "rg2", width, width, 1.5)
        vec(p + "rg2.b", width, 0.3, 0.5)
        lp = p + "mlp."
        if f["kind"] == "dense":
            lin(lp + "up", f["ff"], width, 1.2)
            lin(lp + "down", width, f["ff"])
            W[lp + "act"] = torch.tensor([0.7, -0.4, 0.5, 0.2]).to(
                torch.bfloat16)
            continue
        r, ff = f["router"], f["expert"]["ff"]
        for e in range(r["experts"]):
            lin(f"{lp}e{e}.gate", ff, width, 1.5)
            lin(f"{lp}e{e}.up", ff, width, 1.5)
            lin(f"{lp}e{e}.down", width, ff, 1.5)
        W[lp + "table"] = torch.rand(vocab, r["experts"], generator=g).topk(
            r["top"], dim=1).indices.to(torch.int32)
    return W
