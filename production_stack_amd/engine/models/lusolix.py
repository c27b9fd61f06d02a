"""Lusolix: a decoder over an fp32 residual stream with learned positions,
windowed latent attention in every layer, gated residual branches, an input
convolution ahead of the mixer, and feed-forwards that are dense with a
polynomial norm activation or routed by a table of token ids.

With ln(x; w, b) = (x - mean) / sqrt(var + eps) * w + b, c(h) = h + conv(h)
(causal, per channel, `taps` taps) and m the residual multiplier a layer does
    h = ln(x; w1, b1);  x <- x + m * sigmoid(R1 h + r1) * attention(c(h))
    h = ln(x; w2, b2);  x <- x + m * sigmoid(R2 h + r2) * ff(h)
(the second line in layers with a feed-forward). The embedding output is
embed[token] + pos[position]; logits are embed ln(x; w_f, b_f).

attention: queries W_uq rms(W_dq h), keys and values expanded from one
cached latent rms(W_dkv h) per token, one rotated key part shared by the
heads, trailing window, every head's output times sigmoid(W_g h)_head.
Dense ff: W_down P(W_up h), P(z) = c0 N(z) + c1 N(z^2) + c2 N(z^3) + c3 with
N dividing by the row's root mean square. Routed ff: the mean of the silu
gated experts that a table names for the token id; there is no router.

Per layer the GPU work is: boundary kernel (gate, scale and add the previous
sublayer's output to the stream in fp32, layer norm, input convolution;
writes both h and c(h)) -> one GEMM over query latent | key latent | rotated
key | head gates, one GEMM for the residual gate -> query latent norm -> W_uq
-> fold into the latent space, latent norm + rotary + cache append ->
attention -> expansion, head gates -> W_o -> boundary kernel -> up |
residual gate in one GEMM, polynomial norm, down (or the grouped experts) ->
the next layer's boundary kernel. All table-routed layers of a step are
planned by one launch at its start, since their routing depends on the token
ids alone.

Numerics: the stream, all norms and the convolution with its state, rotary
angles, attention scores / weights, gates' sigmoids and the experts' weighted
sum are fp32; projections and activations run in the serving dtype.

config.json layout read here: architecture, vocab, width, max_positions,
norm{eps}, canon{taps}, residual_mult, layers[i] = {type, mixer{heads, dim,
rot_dim, vdim, kv_rank, q_rank, scale, mask{size}, rot{base, dims}},
mlp{kind, ff | expert{ff}, router{experts, top}}|null}. Checkpoint names:
embed, pos, final.norm(.b), l<i>.norm1(.b) / norm2(.b) / canon1 / rg1(.b) /
rg2(.b), l<i>.mix.{dq, dq.norm, uq, dkv, dkv.norm, uk, uv, g, o},
l<i>.mlp.{up, down, act} or l<i>.mlp.{table, e<j>.gate, e<j>.up, e<j>.down}.
"""

from __future__ import annotations

import json
import os
from typing import List, Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from production_stack_amd import ops
from production_stack_amd.engine.config import (
    LayerSpec,
    MixerSpec,
    MlpSpec,
    ModelConfig,
)
from production_stack_amd.engine.models.ffn import (
    GatedMLP,
    SparseMoE,
    TablePlans,
)
from production_stack_amd.engine.models.mixers import build_mixer
from production_stack_amd.ops import gemm_policy

ARCHITECTURE = "Lusolix"


# ---------------------------------------------------------------------------
# configuration
# ---------------------------------------------------------------------------
def _mixer_spec(kind: str, m: dict) -> MixerSpec:
    if kind != "latent_attention":
        raise ValueError(f"unknown layer type {kind!r}")
    rot = m.get("rot") or {}
    mask = m.get("mask") or {}
    return MixerSpec(
        kind="latent_attention", heads=int(m["heads"]), kv_heads=1,
        dim=int(m["dim"]), vdim=int(m.get("vdim", m["dim"])),
        kv_rank=int(m["kv_rank"]), q_rank=int(m["q_rank"]),
        rot_dim=int(m["rot_dim"]),
        rot_dims=int(rot.get("dims", m["rot_dim"])),
        rot_base=float(rot.get("base", 10000.0)), scale=float(m["scale"]),
        window=int(mask.get("size", 0)), head_gate=True, rope=True)


def _mlp_spec(m: Optional[dict], vocab: int) -> Optional[MlpSpec]:
    if m is None:
        return None
    if m["kind"] == "dense":
        return MlpSpec(kind="dense", ff=int(m["ff"]), act="poly_norm",
                       gated=False)
    if m["kind"] == "moe":
        r = m["router"]
        return MlpSpec(
            kind="moe", ff=int(m["expert"]["ff"]), act="silu",
            experts=int(r["experts"]), top=int(r["top"]), score="table",
            renormalize=False, table_rows=vocab)
    raise ValueError(f"unknown mlp kind {m['kind']!r}")


def config_from_json(cfg: dict, name: str = "lusolix") -> ModelConfig:
    taps = int((cfg.get("canon") or {}).get("taps", 0))
    vocab = int(cfg["vocab"])
    specs: List[LayerSpec] = [
        LayerSpec(mixer=_mixer_spec(layer["type"], layer["mixer"]),
                  mlp=_mlp_spec(layer.get("mlp"), vocab), parallel=False,
                  norm="layer", input_conv=taps, mlp_conv=False,
                  residual_gate=True)
        for layer in cfg["layers"]]
    mixers = [s.mixer for s in specs]
    ffs = [s.mlp.ff for s in specs if s.mlp is not None]
    positions = int(cfg["max_positions"])
    return ModelConfig(
        name=name, family="lusolix", hidden_size=int(cfg["width"]),
        num_layers=len(specs),
        num_q_heads=max([m.heads for m in mixers], default=1),
        num_kv_heads=1,
        head_dim=max([m.dim + m.rot_dim for m in mixers], default=1),
        intermediate_size=max(ffs, default=0), vocab_size=vocab,
        max_position=positions, learned_positions=positions,
        rms_norm_eps=float(cfg["norm"]["eps"]), layer_specs=specs,
        residual_mult=float(cfg.get("residual_mult", 1.0)),
        tie_word_embeddings=True,
        # no BOS/EOS convention in this design: never stop on a token id
        bos_token_id=0, eos_token_id=-1)


def config_from_dir(path: str) -> ModelConfig:
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    return config_from_json(cfg, name=os.path.basename(
        os.path.normpath(path)) or "lusolix")


# ---------------------------------------------------------------------------
# model
# ---------------------------------------------------------------------------
class LusolixLayer(nn.Module):
    def __init__(self, width: int, spec: LayerSpec, eps: float,
                 dtype: torch.dtype, max_pos: int) -> None:
        super().__init__()
        if (spec.parallel or spec.norm != "layer" or spec.mlp_conv
                or not spec.residual_gate):
            raise NotImplementedError(
                "sequential gated sublayers behind layer norms, with a "
                "convolution on the mixer's input only")
        self.spec = spec
        self.width = width
        f32 = torch.float32
        K = spec.input_conv

        def vec():
            return nn.Parameter(torch.empty(width, dtype=f32))

        def square():
            return nn.Parameter(torch.empty(width, width, dtype=dtype))

        self.norm1, self.norm1_b = vec(), vec()
        self.conv1 = (nn.Parameter(torch.empty(width, K, dtype=f32))
                      if K else None)
        self.mixer = build_mixer(width, spec.mixer, eps, dtype, max_pos)
        self.rg1, self.rg1_b = square(), vec()
        self.mlp = None
        self.norm2 = self.norm2_b = self.rg2 = self.rg2_b = None
        self._fused = None
        if spec.mlp is not None:
            self.norm2, self.norm2_b = vec(), vec()
            self.rg2, self.rg2_b = square(), vec()
            self.mlp = (
                GatedMLP(width, spec.mlp.ff, spec.mlp.act, spec.mlp.limit,
                         dtype, spec.mlp.gated, eps)
                if spec.mlp.kind == "dense"
                else SparseMoE(width, spec.mlp, dtype))

    def _apply(self, fn, *a, **kw):
        # the fused weight is a plain tensor rebuilt after a move
        self._fused = None
        return super()._apply(fn, *a, **kw)

    def fused_ff(self) -> torch.Tensor:
        """A dense feed-forward's up rows | residual gate rows as one
        weight; the parts become views of it."""
        w = self._fused
        if w is None:
            n = self.mlp.gate_up.shape[0]
            w = torch.cat([self.mlp.gate_up.data, self.rg2.data],
                          dim=0).contiguous()
            self.mlp.gate_up.data, self.rg2.data = w[:n], w[n:]
            self._fused = w
        return w

    def feed_forward(self, h: torch.Tensor, small: Optional[bool], plan):
        """(feed-forward output, residual gate before bias and sigmoid)."""
        if self.spec.mlp.kind == "dense":
            proj = gemm_policy.linear(h, self.fused_ff())
            n = self.mlp.in_rows
            return self.mlp.forward_from_proj(proj[:, :n]), proj[:, n:]
        return (self.mlp(h, small, plan), gemm_policy.linear(h, self.rg2))

    def cache_shape(self):
        """mixer cache, then the convolution's tail."""
        parts = [self.mixer.cache_shape()]
        K = self.spec.input_conv
        if K:
            parts.append(("slots", (K - 1, self.width), torch.float32))
        return ("multi", parts)


class LusolixForCausalLM(nn.Module):
    # per-step metadata this family needs from the runner
    needs_seq_meta = True
    # single-token steps run planned experts without a host read, so they
    # replay a hipGraph
    supports_decode_graph = True

    def __init__(self, cfg: ModelConfig, tp: int = 1, pp_rank: int = 0,
                 pp_size: int = 1, dtype: torch.dtype = torch.bfloat16
                 ) -> None:
        super().__init__()
        if tp != 1 or pp_size != 1:
            raise NotImplementedError(
                "Lusolix runs on one GPU per replica (no TP/PP sharding of "
                "the latent cache yet)")
        self.cfg = cfg
        self.tp = 1
        self.dtype = dtype
        W = cfg.hidden_size
        self.embed = nn.Parameter(torch.empty(cfg.vocab_size, W,
                                              dtype=dtype))
        self.pos = nn.Parameter(torch.empty(cfg.learned_positions, W,
                                            dtype=dtype))
        self.layers = nn.ModuleList(
            LusolixLayer(W, spec, cfg.rms_norm_eps, dtype, cfg.max_position)
            for spec in cfg.layer_specs)
        self.final_norm = nn.Parameter(torch.empty(W, dtype=torch.float32))
        self.final_norm_b = nn.Parameter(torch.empty(W,
                                                     dtype=torch.float32))
        # layers whose experts a table names, and their place in the plans
        self.table_layers = [i for i, s in enumerate(cfg.layer_specs)
                             if s.mlp is not None and s.mlp.kind == "moe"]
        self.plans = TablePlans([self.layers[i].mlp
                                 for i in self.table_layers])
        # optional debugging tap: called with (layer index, fp32 residual
        # stream after that layer)
        self.residual_hook = None

    # ---- cache geometry ------------------------------------------------
    @property
    def num_local_layers(self) -> int:
        return len(self.layers)

    def cache_shapes(self):
        return [layer.cache_shape() for layer in self.layers]

    def kv_bytes_per_block(self, block_size: int) -> int:
        esz = 4 if self.dtype == torch.float32 else 2
        return sum(d[1] * block_size * d[2] * esz
                   for _, parts in self.cache_shapes()
                   for d in parts if d[0] == "paged")

    def state_bytes_per_seq(self) -> int:
        return sum(d[1][0] * d[1][1] * 4 for _, parts in self.cache_shapes()
                   for d in parts if d[0] == "slots")

    def gemm_weights(self):
        """One weight per distinct projection shape of the stack (for the
        per-shape GEMM choice at decode batch sizes)."""
        seen, out = set(), []
        for layer in self.layers:
            mx = layer.mixer
            cands = [mx.in_proj, mx.uq, mx.out_weight, layer.rg1]
            if layer.mlp is not None:
                cands += ([layer.fused_ff(), layer.mlp.down]
                          if layer.spec.mlp.kind == "dense"
                          else [layer.rg2])
            for w in cands:
                if w is not None and w.dim() == 2 and w.is_contiguous() \
                        and tuple(w.shape) not in seen:
                    seen.add(tuple(w.shape))
                    out.append(w)
        return out

    # ---- weights -------------------------------------------------------
    @torch.no_grad()
    def random_init(self, seed: int = 0) -> None:
        dev = self.embed.device
        gen = torch.Generator(device=dev).manual_seed(seed)
        for name, p in self.named_parameters():
            last = name.rsplit(".", 1)[-1]
            if last == "table":
                # distinct experts per row
                V, top = p.shape
                E = self.layers[int(name.split(".")[1])].spec.mlp.experts
                p.copy_(torch.rand(V, E, generator=gen, device=dev).topk(
                    top, dim=1).indices)
            elif last in ("norm1", "norm2", "final_norm", "q_norm",
                          "latent_norm"):
                p.normal_(1.0, 0.1, generator=gen)
            elif last in ("norm1_b", "norm2_b", "final_norm_b"):
                p.normal_(0.0, 0.1, generator=gen)
            elif last in ("rg1_b", "rg2_b"):
                p.normal_(0.0, 0.5, generator=gen)
            elif last == "conv1":
                p.normal_(0.0, 0.3, generator=gen)
            elif last == "poly":
                p.normal_(0.3, 0.1, generator=gen)
            elif last == "embed":
                p.normal_(0.0, 1.0, generator=gen)
            elif last == "pos":
                p.normal_(0.0, 0.3, generator=gen)
            elif last == "uv":
                p.normal_(0.0, p.shape[1] ** -0.5, generator=gen)
            else:
                p.normal_(0.0, p.shape[-1] ** -0.5, generator=gen)
        self._drop_fused()

    def _drop_fused(self) -> None:
        self.plans.drop()
        for layer in self.layers:
            layer._fused = None

    @torch.no_grad()
    def load_weights(self, path: str) -> None:
        from safetensors import safe_open

        f = safe_open(os.path.join(path, "model.safetensors"),
                      framework="pt", device="cpu")

        def check(t, param, name):
            if tuple(t.shape) != tuple(param.shape):
                raise ValueError(
                    f"{name}: checkpoint shape {tuple(t.shape)} != "
                    f"{tuple(param.shape)}")

        def put(param, name, shape=None):
            t = f.get_tensor(name)
            if shape is not None and tuple(t.shape) == shape:
                t = t.view(param.shape)
            check(t, param, name)
            param.copy_(t.to(param.dtype))

        def cat(param, names):
            t = torch.cat([f.get_tensor(n) for n in names], dim=0)
            check(t, param, names)
            param.copy_(t.to(param.dtype))

        put(self.embed, "embed")
        put(self.pos, "pos")
        put(self.final_norm, "final.norm")
        put(self.final_norm_b, "final.norm.b")
        for i, layer in enumerate(self.layers):
            pre = f"l{i}."
            put(layer.norm1, pre + "norm1")
            put(layer.norm1_b, pre + "norm1.b")
            if layer.conv1 is not None:
                put(layer.conv1, pre + "canon1")
            put(layer.rg1, pre + "rg1")
            put(layer.rg1_b, pre + "rg1.b")
            mx, mp = layer.mixer, pre + "mix."
            cat(mx.in_proj, [mp + "dq", mp + "dkv", mp + "g"])
            put(mx.q_norm, mp + "dq.norm")
            put(mx.uq, mp + "uq")
            put(mx.latent_norm, mp + "dkv.norm")
            put(mx.uk, mp + "uk", (mx.H * mx.D, mx.L))
            mx.load_uv(f.get_tensor(mp + "uv"))
            put(mx.out_weight, mp + "o")
            ml, lp = layer.mlp, pre + "mlp."
            if ml is None:
                continue
            put(layer.norm2, pre + "norm2")
            put(layer.norm2_b, pre + "norm2.b")
            put(layer.rg2, pre + "rg2")
            put(layer.rg2_b, pre + "rg2.b")
            if layer.spec.mlp.kind == "dense":
                put(ml.gate_up, lp + "up")
                put(ml.down, lp + "down")
                put(ml.poly, lp + "act")
            else:
                ml.load_table(f.get_tensor(lp + "table"))
                for e in range(ml.spec.experts):
                    ep = f"{lp}e{e}."
                    cat(ml.experts_gate_up[e], [ep + "gate", ep + "up"])
                    put(ml.experts_down[e], ep + "down")
        self._drop_fused()

    # ---- forward -------------------------------------------------------
    @torch.no_grad()
    def forward(self, token_ids: torch.Tensor, meta, caches,
                residual=None) -> torch.Tensor:
        cfg = self.cfg
        eps, dt, m = cfg.rms_norm_eps, self.dtype, cfg.residual_mult
        x = ops.embed_scale(token_ids, self.embed, 1.0, self.pos,
                            meta.positions)                   # fp32 [T, W]
        # steps of single tokens only must not read from the device
        small = True if getattr(meta, "num_prefill_tokens", None) == 0 \
            else None
        plans = {}
        if self.table_layers:
            on_host = (small is None and token_ids.shape[0]
                       > SparseMoE.GROUPED_MAX_ROWS)
            plans = dict(zip(self.table_layers,
                             self.plans.plan(token_ids, on_host)))
        shared: dict = {}
        hook = self.residual_hook
        # the sublayer output not yet in the stream, with its gate; the
        # next boundary kernel adds it in fp32
        pend, gate = [], None

        def boundary(norm, bias, conv, tail, plain):
            return ops.add_layer_norm_conv32(
                x, pend, [m] * len(pend), norm, bias, eps, conv, tail,
                meta.seq_rows, dt, gate, plain)

        for i, (layer, cache) in enumerate(zip(self.layers, caches)):
            K = layer.spec.input_conv
            hc, h = boundary(layer.norm1, layer.norm1_b, layer.conv1,
                             cache[1] if K else None, True)
            mx = layer.mixer
            o = mx(hc, meta, cache[0], shared)
            pend = [gemm_policy.linear(o, mx.out_weight)]
            gate = (gemm_policy.linear(h, layer.rg1), layer.rg1_b)
            if layer.mlp is not None:
                h = boundary(layer.norm2, layer.norm2_b, None, None, False)
                y, z = layer.feed_forward(h, small, plans.get(i))
                pend, gate = [y], (z, layer.rg2_b)
            if hook is not None:
                x.add_(pend[0].float() * torch.sigmoid(
                    gate[0].float() + gate[1]), alpha=m)
                pend, gate = [], None
                hook(i, x)
        return boundary(self.final_norm, self.final_norm_b, None, None,
                        False)

    @torch.no_grad()
    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return F.linear(hidden, self.embed).float()
