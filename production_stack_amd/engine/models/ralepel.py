"""Ralepel: a decoder over an fp32 residual stream whose sublayers read the
stream itself and are normalised on their outputs only; windowed attention
whose keys are its values, latent attention (some layers on an earlier
layer's cache), dense or routed feed-forwards.

With rms(y; w) = y / sqrt(mean(y^2) + eps) * w a layer does
    x <- x + rms(mixer(x); w1);  x <- x + rms(ff(x); w2)
(the second part in layers with a feed-forward). The stream starts as
embed[token]; logits are head rms(x; w_f).

attention: q = W_q x + b_q, v = W_k x + b_k, k = v; query and key heads over
their root mean square; score_ij = scale q_i k_j - slope_h (i - j) over the
trailing window, softmax with a learned sink per head, output bias.
latent_attention: queries [unrotated | rotated] per head, one cached latent
rms(W_dkv x) and one rotated key part per token, keys and values expanded per
head, half-split rotary pairs, plain causal softmax; `kv_from` layers read
another layer's cache through their own up-projections.
Routed ff: softmax over the `top` largest biased router logits, silu-gated
experts, plus a shared expert times the sigmoid of one projected number.

Per layer the GPU work is: one GEMM over query | key with their biases ->
query norm and cache append (keys as projected, their 1/rms beside them) ->
attention -> W_o with its bias -> boundary kernel (output norm, fp32 addition,
next sublayer's input) -> feed-forward -> boundary kernel. Latent layers:
query | latent | rotated key in one GEMM, then as in LatentAttention; layers
on one cache gather its rows once per step.

Numerics: the stream, all norms, rotary angles, attention scores / weights,
router logits and weights, the shared expert's sigmoid and the experts'
weighted sum are fp32; projections and activations run in the serving dtype
(a sublayer's input is the stream rounded to it).

config.json layout read here: architecture, vocab, width, norm{eps},
layers[i] = {type, mixer{heads, dim, vdim, scale, kv_heads, mask{size} |
rot_dim, kv_rank, rot{base, dims}, kv_from}, mlp{kind, ff | expert{ff},
router{experts, top}, shared{ff}}|null}. Checkpoint names: embed, head,
final.norm, l<i>.norm1 / norm2, l<i>.mix.{q(.b), k(.b), sink, o(.b)} or
l<i>.mix.{q, dkv, dkv.norm, uk, uv, o}, l<i>.mlp.{gate, up, down} or
l<i>.mlp.{router(.b), e<j>.gate / up / down, shared.gate / up / down / sg}.
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
from production_stack_amd.engine.models.ffn import GatedMLP, SparseMoE
from production_stack_amd.engine.models.mixers import build_mixer
from production_stack_amd.ops import gemm_policy

ARCHITECTURE = "Ralepel"
# rotary positions are computed, so this only sizes the angle tables; the
# engine's max_model_len raises it where needed
DEFAULT_MAX_POSITION = 8192


# ---------------------------------------------------------------------------
# configuration
# ---------------------------------------------------------------------------
def _mixer_spec(kind: str, m: dict) -> MixerSpec:
    dim, scale = int(m["dim"]), float(m["scale"])
    window = int((m.get("mask") or {}).get("size", 0))
    if kind == "attention":
        if int(m.get("vdim", dim)) != dim:
            raise ValueError(
                "attention: the keys are the values, vdim must equal dim")
        return MixerSpec(
            kind="attention", heads=int(m["heads"]),
            kv_heads=int(m.get("kv_heads", m["heads"])), dim=dim, vdim=dim,
            scale=scale, window=window, sink=True, learned_sink=True,
            bias=True, out_bias=True, rope=False, key_values=True,
            unit_qk=True, distance_bias=True)
    if kind == "latent_attention":
        rot, rot_dim = m["rot"], int(m["rot_dim"])
        src = m.get("kv_from")
        return MixerSpec(
            kind="latent_attention", heads=int(m["heads"]), kv_heads=1,
            dim=dim, vdim=int(m.get("vdim", dim)),
            kv_rank=int(m["kv_rank"]), rot_dim=rot_dim,
            rot_dims=int(rot.get("dims", rot_dim)),
            rot_base=float(rot["base"]), rot_layout="half", scale=scale,
            window=window, rope=True,
            kv_from=int(src) if src is not None else None)
    raise ValueError(f"unknown layer type {kind!r}")


def _mlp_spec(m: Optional[dict]) -> Optional[MlpSpec]:
    if m is None:
        return None
    if m["kind"] == "dense":
        return MlpSpec(kind="dense", ff=int(m["ff"]), act="silu")
    if m["kind"] == "moe":
        r, shared = m["router"], m.get("shared")
        return MlpSpec(
            kind="moe", ff=int(m["expert"]["ff"]), act="silu",
            experts=int(r["experts"]), top=int(r["top"]), score="softmax",
            renormalize=True, router_bias=True,
            shared_ff=int(shared["ff"]) if shared else 0)
    raise ValueError(f"unknown mlp kind {m['kind']!r}")


def _check_sources(specs: List[LayerSpec]) -> None:
    """kv_from names an earlier latent layer with a cache of its own and the
    same rows."""
    for i, s in enumerate(specs):
        m = s.mixer
        if m.kv_from is None:
            continue
        src = specs[m.kv_from].mixer if 0 <= m.kv_from < i else None
        if src is None or src.kind != m.kind or src.kv_from is not None or (
                src.kv_rank, src.rot_dim, src.rot_dims, src.rot_base) != (
                m.kv_rank, m.rot_dim, m.rot_dims, m.rot_base):
            raise ValueError(
                f"layer {i}: kv_from {m.kv_from} is no earlier latent layer "
                "with rows of the same layout")


def config_from_json(cfg: dict, name: str = "ralepel") -> ModelConfig:
    specs: List[LayerSpec] = [
        LayerSpec(mixer=_mixer_spec(layer["type"], layer["mixer"]),
                  mlp=_mlp_spec(layer.get("mlp")), parallel=False,
                  post_norm=True, pre_norm=False)
        for layer in cfg["layers"]]
    _check_sources(specs)
    mixers = [s.mixer for s in specs]
    ffs = [max(s.mlp.ff, s.mlp.shared_ff) for s in specs
           if s.mlp is not None]
    return ModelConfig(
        name=name, family="ralepel", hidden_size=int(cfg["width"]),
        num_layers=len(specs),
        num_q_heads=max([m.heads for m in mixers], default=1),
        num_kv_heads=max([m.kv_heads for m in mixers], default=1),
        head_dim=max([m.dim + m.rot_dim for m in mixers], default=1),
        intermediate_size=max(ffs, default=0),
        vocab_size=int(cfg["vocab"]),
        max_position=int(cfg.get("max_position", DEFAULT_MAX_POSITION)),
        rms_norm_eps=float(cfg["norm"]["eps"]), layer_specs=specs,
        # no BOS/EOS convention in this design: never stop on a token id
        bos_token_id=0, eos_token_id=-1)


def config_from_dir(path: str) -> ModelConfig:
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    return config_from_json(cfg, name=os.path.basename(
        os.path.normpath(path)) or "ralepel")


# ---------------------------------------------------------------------------
# model
# ---------------------------------------------------------------------------
class RalepelLayer(nn.Module):
    def __init__(self, width: int, spec: LayerSpec, eps: float,
                 dtype: torch.dtype, max_pos: int) -> None:
        super().__init__()
        if spec.parallel or spec.pre_norm or not spec.post_norm:
            raise NotImplementedError(
                "sequential sublayers, normalised on their outputs only")
        self.spec = spec

        def vec():
            return nn.Parameter(torch.empty(width, dtype=torch.float32))

        self.norm1 = vec()
        self.mixer = build_mixer(width, spec.mixer, eps, dtype, max_pos)
        self.mlp = self.norm2 = None
        if spec.mlp is not None:
            self.norm2 = vec()
            self.mlp = (
                GatedMLP(width, spec.mlp.ff, spec.mlp.act, spec.mlp.limit,
                         dtype)
                if spec.mlp.kind == "dense"
                else SparseMoE(width, spec.mlp, dtype))

    def mix(self, h: torch.Tensor, meta, cache, shared: dict):
        o = self.mixer(h, meta, cache, shared)
        if self.spec.mixer.kind == "attention":
            return self.mixer.project(o)
        return gemm_policy.linear(o, self.mixer.out_weight)

    def feed_forward(self, h: torch.Tensor, small: Optional[bool]):
        if self.spec.mlp.kind == "dense":
            return self.mlp(h)
        return self.mlp(h, small)


class RalepelForCausalLM(nn.Module):
    # per-step metadata this family needs from the runner
    needs_seq_meta = True
    # single-token steps route and run their experts without a host read, so
    # they replay a hipGraph
    supports_decode_graph = True

    def __init__(self, cfg: ModelConfig, tp: int = 1, pp_rank: int = 0,
                 pp_size: int = 1, dtype: torch.dtype = torch.bfloat16
                 ) -> None:
        super().__init__()
        if tp != 1 or pp_size != 1:
            raise NotImplementedError(
                "Ralepel runs on one GPU per replica (no TP/PP sharding of "
                "the shared latent cache yet)")
        self.cfg = cfg
        self.tp = 1
        self.dtype = dtype
        W = cfg.hidden_size
        self.embed = nn.Parameter(torch.empty(cfg.vocab_size, W,
                                              dtype=dtype))
        self.layers = nn.ModuleList(
            RalepelLayer(W, spec, cfg.rms_norm_eps, dtype, cfg.max_position)
            for spec in cfg.layer_specs)
        self.final_norm = nn.Parameter(torch.empty(W, dtype=torch.float32))
        self.lm_head = nn.Parameter(torch.empty(cfg.vocab_size, W,
                                                dtype=dtype))
        # optional debugging tap: called with (layer index, fp32 residual
        # stream after that layer)
        self.residual_hook = None

    # ---- cache geometry ------------------------------------------------
    @property
    def num_local_layers(self) -> int:
        return len(self.layers)

    def cache_shapes(self):
        return [layer.mixer.cache_shape() for layer in self.layers]

    def kv_bytes_per_block(self, block_size: int) -> int:
        esz = 4 if self.dtype == torch.float32 else 2
        n = 0
        for d in self.cache_shapes():
            if d[0] == "keyval":
                n += d[1] * (d[2] * esz + 4)
            elif d[0] == "paged":
                n += d[1] * d[2] * esz
        return n * block_size

    def state_bytes_per_seq(self) -> int:
        return 0

    def gemm_weights(self):
        """One weight per distinct projection shape of the stack (for the
        per-shape GEMM choice at decode batch sizes)."""
        seen, out = set(), []
        for layer in self.layers:
            mx, ml = layer.mixer, layer.mlp
            # the attention layers' projections have biases, which only the
            # vendor GEMM adds in its accumulator
            cands = [] if layer.spec.mixer.kind == "attention" else [
                *mx.in_params(), mx.out_weight]
            if ml is not None:
                if layer.spec.mlp.kind == "dense":
                    cands += [ml.gate_up, ml.down]
                elif ml.shared is not None:
                    cands += [ml.fused_in(), ml.shared.down]
            for w in cands:
                if w.is_contiguous() and tuple(w.shape) not in seen:
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
            if last in ("norm1", "norm2", "final_norm", "latent_norm"):
                p.normal_(1.0, 0.1, generator=gen)
            elif last in ("qkv_bias", "out_bias", "router_bias"):
                p.normal_(0.0, 0.3, generator=gen)
            elif last in ("sink_vals", "embed"):
                p.normal_(0.0, 1.0, generator=gen)
            elif last == "uv":
                p.normal_(0.0, p.shape[1] ** -0.5, generator=gen)
            else:
                p.normal_(0.0, p.shape[-1] ** -0.5, generator=gen)
        self._drop_fused()

    def _drop_fused(self) -> None:
        for layer in self.layers:
            if layer.spec.mixer.kind == "latent_attention":
                layer.mixer._unfolded = None
            if isinstance(layer.mlp, SparseMoE):
                layer.mlp._fused_in = None

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
        put(self.lm_head, "head")
        put(self.final_norm, "final.norm")
        for i, layer in enumerate(self.layers):
            pre = f"l{i}."
            put(layer.norm1, pre + "norm1")
            mx, mp = layer.mixer, pre + "mix."
            if layer.spec.mixer.kind == "attention":
                cat(mx.qkv, [mp + "q", mp + "k"])
                cat(mx.qkv_bias, [mp + "q.b", mp + "k.b"])
                put(mx.sink_vals, mp + "sink")
                put(mx.out_bias, mp + "o.b")
            else:
                names = [mp + "q"]
                if mx.latent_norm is not None:
                    names.append(mp + "dkv")
                    put(mx.latent_norm, mp + "dkv.norm")
                cat(mx.in_proj, names)
                put(mx.uk, mp + "uk", (mx.H * mx.D, mx.L))
                mx.load_uv(f.get_tensor(mp + "uv"))
            put(mx.out_weight, mp + "o")
            ml, lp = layer.mlp, pre + "mlp."
            if ml is None:
                continue
            put(layer.norm2, pre + "norm2")
            if layer.spec.mlp.kind == "dense":
                cat(ml.gate_up, [lp + "gate", lp + "up"])
                put(ml.down, lp + "down")
                continue
            put(ml.router, lp + "router")
            put(ml.router_bias, lp + "router.b")
            for e in range(ml.spec.experts):
                ep = f"{lp}e{e}."
                cat(ml.experts_gate_up[e], [ep + "gate", ep + "up"])
                put(ml.experts_down[e], ep + "down")
            if ml.shared is not None:
                sp = lp + "shared."
                cat(ml.shared.gate_up, [sp + "gate", sp + "up"])
                put(ml.shared.down, sp + "down")
                put(ml.shared_gate, sp + "sg")
        self._drop_fused()

    # ---- forward -------------------------------------------------------
    @torch.no_grad()
    def forward(self, token_ids: torch.Tensor, meta, caches,
                residual=None) -> torch.Tensor:
        eps, dt = self.cfg.rms_norm_eps, self.dtype
        x = ops.embed_scale(token_ids, self.embed, 1.0)       # fp32 [T, W]
        # the stream's rounding to the serving dtype: the row itself
        h = F.embedding(token_ids, self.embed)
        # steps of single tokens only must not read from the device
        small = True if getattr(meta, "num_prefill_tokens", None) == 0 \
            else None
        shared: dict = {}
        hook = self.residual_hook
        last = len(self.layers) - 1
        for i, (layer, cache) in enumerate(zip(self.layers, caches)):
            w_out = self.final_norm if i == last else None
            y = layer.mix(h, meta, cache, shared)
            w = layer.norm1
            if layer.mlp is not None:
                h = ops.post_norm_add_norm32(x, y, w, None, eps, dt)
                y, w = layer.feed_forward(h, small), layer.norm2
            h = ops.post_norm_add_norm32(x, y, w, w_out, eps, dt)
            if hook is not None:
                hook(i, x)
        return h

    @torch.no_grad()
    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return F.linear(hidden, self.lm_head).float()
