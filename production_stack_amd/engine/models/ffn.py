"""Feed-forward building blocks shared by the model families.

  * route():       fp32 router with softmax or sigmoid scores, top-k and
                   optional renormalisation of the chosen weights (torch
                   ops; SparseMoE uses the one-kernel ops.moe_route);
  * sparse_moe():  expert dispatch: rows are sorted by expert once (one
                   host read of the per-expert counts per call) and every
                   expert runs the dense GEMM path over its slice, with the
                   routing weight on the expert's output or on its input;
  * ExpertPlan:    a step's routed rows sorted by expert (ops.expert_plan);
                   SparseMoE runs the experts over them in one grouped
                   kernel pair (small batches) or one GEMM pair per expert;
  * GatedMLP / SparseMoE: parameter holders driven by engine.config.MlpSpec,
                   used by the heterogeneous (per-layer spec) models.

The Llama family's Mixtral layers call route()/sparse_moe() too.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Callable, List, Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from production_stack_amd import ops
from production_stack_amd.engine.config import MlpSpec
from production_stack_amd.ops import gemm_policy


def route(x: torch.Tensor, router_w: torch.Tensor, top: int,
          score: str = "softmax", renormalize: bool = True,
          correction: Optional[torch.Tensor] = None, scale: float = 1.0,
          renorm_eps: float = 0.0):
    """Returns (weights fp32 [T, top], expert ids [T, top]). The logits are
    an fp32 product of the (up-cast) activations and router weights.
    correction (fp32 [experts]): added to the softmax scores for the choice
    only, the weights are the plain scores; the chosen weights are divided
    by (their sum + renorm_eps) when renormalize, then multiplied by
    scale."""
    logits = F.linear(x.float(), router_w.float())
    if score == "softmax":
        probs = torch.softmax(logits, dim=-1)
        if correction is not None:
            _, sel = torch.topk(probs + correction, top, dim=-1)
            weights = probs.gather(-1, sel)
        else:
            weights, sel = torch.topk(probs, top, dim=-1)
    elif score == "sigmoid":
        # rank by the logits: the sigmoid is monotonic but saturates to
        # exactly 1.0 in fp32, which would tie large scores
        _, sel = torch.topk(logits, top, dim=-1)
        weights = torch.sigmoid(logits.gather(-1, sel))
    else:
        raise ValueError(f"unknown router score {score!r}")
    if renormalize:
        weights = weights / (weights.sum(dim=-1, keepdim=True) + renorm_eps)
    if scale != 1.0:
        weights = weights * scale
    return weights, sel


def sparse_moe(x: torch.Tensor, weights: torch.Tensor, sel: torch.Tensor,
               n_experts: int,
               expert_fn: Callable[[int, torch.Tensor], torch.Tensor],
               weight_on_input: bool = False,
               out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """sum over chosen experts of  w * expert(x)  (or expert(w * x)).

    expert_fn(e, rows_of_x) -> rows_of_y. `out` (zero-filled [T, width],
    any float dtype) is accumulated into and returned; it defaults to x's
    dtype."""
    T, K = sel.shape
    if out is None:
        out = torch.zeros_like(x)
    flat = sel.reshape(-1)
    order = torch.argsort(flat, stable=True)
    counts = torch.bincount(flat, minlength=n_experts).tolist()
    rows_sorted = torch.div(order, K, rounding_mode="floor")
    w_sorted = weights.reshape(-1)[order]
    start = 0
    for e, n in enumerate(counts):
        if n == 0:
            continue
        rows = rows_sorted[start:start + n]
        w = w_sorted[start:start + n]
        start += n
        xe = x.index_select(0, rows)
        if weight_on_input:
            xe = (xe.float() * w.unsqueeze(-1)).to(x.dtype)
            ye = expert_fn(e, xe)
        elif out.dtype == torch.float32:
            # fp32 accumulator: the fp32 routing weight is applied unrounded
            ye = expert_fn(e, xe).float() * w.unsqueeze(-1)
        else:
            ye = expert_fn(e, xe) * w.to(x.dtype).unsqueeze(-1)
        out.index_add_(0, rows, ye.to(out.dtype))
    return out


def _right(w: torch.Tensor) -> torch.Tensor:
    """[E, N, K] as the right operand [E, K, N] of a batched product: a
    contiguous copy in bfloat16 (a transposed view is not safe there)."""
    t = w.transpose(1, 2)
    return t.contiguous() if w.dtype == torch.bfloat16 else t


@dataclass
class ExpertPlan:
    """Which rows of a step go to which expert. With n = T * top routed
    entries (token t's k-th choice is entry t * top + k), stably sorted by
    router output: output o owns the sorted entries offs[o] .. offs[o + 1],
    rows[i] is the token of sorted entry i and pos[t * top + k] the sorted
    place of an entry (int32 device tensors). weights fp32 [T, top] (None:
    every entry weighs `weight`); sel int64 [T, top] (None where no output
    beyond the experts exists). counts: entries per output on the host,
    where a caller has read them."""

    offs: torch.Tensor
    rows: torch.Tensor
    pos: torch.Tensor
    top: int
    weights: Optional[torch.Tensor] = None
    weight: float = 1.0
    sel: Optional[torch.Tensor] = None
    counts: Optional[List[int]] = None

    def host_counts(self) -> List[int]:
        if self.counts is None:
            offs = self.offs.tolist()
            self.counts = [b - a for a, b in zip(offs, offs[1:])]
        return self.counts

    def dense(self, n_out: int) -> torch.Tensor:
        """fp32 [T, n_out]: the weights at the chosen outputs, else 0."""
        n = self.pos.numel()
        wm = torch.zeros((n // self.top, n_out), dtype=torch.float32,
                         device=self.pos.device)
        # sorted place -> output: the number of segments that end before it
        out_of = torch.searchsorted(self.offs[1:].contiguous(), self.pos,
                                    right=True).view(-1, self.top)
        w = (self.weights if self.weights is not None else
             torch.full_like(out_of, self.weight, dtype=torch.float32))
        return wm.scatter_(1, out_of, w)


class GatedMLP(nn.Module):
    """down(act(gate x) * up x); gate and up are one fused projection. The
    fused in-projection may be run by the caller together with other
    consumers of the same input (see in_params / forward_from_proj).
    gated False: down(act(up x)), `gate_up` then holds the up rows only.
    act "poly_norm" (not gated) has four learned coefficients `poly` and
    normalises with `eps`."""

    def __init__(self, width: int, ff: int, act: str, limit: float,
                 dtype: torch.dtype, gated: bool = True,
                 eps: float = 1e-5) -> None:
        super().__init__()
        self.poly, self.eps = None, eps
        if act == "poly_norm":
            if gated:
                raise ValueError("poly_norm has no gate branch")
            self.poly = nn.Parameter(torch.empty(4, dtype=torch.float32))
        self.ff, self.act, self.limit, self.gated = ff, act, limit, gated
        self.in_rows = (2 if gated else 1) * ff
        self.gate_up = nn.Parameter(
            torch.empty(self.in_rows, width, dtype=dtype))
        self.down = nn.Parameter(torch.empty(width, ff, dtype=dtype))

    def in_params(self):
        return [self.gate_up]

    def inner(self, proj: torch.Tensor,
              out: Optional[torch.Tensor] = None) -> torch.Tensor:
        """proj [T, 2*ff] = gate | up (or [T, ff] without a gate)  ->
        activation [T, ff]."""
        if self.poly is not None:
            return ops.poly_norm(proj, self.poly, self.eps, out=out)
        if not self.gated:
            return ops.gated_act(proj, None, self.act, self.limit, out=out)
        return ops.gated_act(proj[:, :self.ff], proj[:, self.ff:], self.act,
                             self.limit, out=out)

    def forward_from_proj(self, proj: torch.Tensor) -> torch.Tensor:
        return gemm_policy.linear(self.inner(proj), self.down)

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        return self.forward_from_proj(gemm_policy.linear(x, self.gate_up))


class SparseMoE(nn.Module):
    """Routed experts (+ optional always-on shared expert scaled by a
    per-token sigmoid gate), configured by an MlpSpec. The router may have
    `identity` outputs beyond the experts: choosing one of them returns
    the (weighted) input itself. score "table": `table` [table_rows, top]
    names every token id's experts, there is no router, and the caller
    passes the step's plan (table_plans)."""

    def __init__(self, width: int, spec: MlpSpec, dtype: torch.dtype) -> None:
        super().__init__()
        self.spec = spec
        E, ff = spec.experts, spec.ff
        self.router = self.table = None
        if spec.score == "table":
            self.table = nn.Parameter(
                torch.empty(spec.table_rows, spec.top, dtype=torch.int32),
                requires_grad=False)
        else:
            self.router = nn.Parameter(
                torch.empty(E + spec.identity, width, dtype=dtype))
        self.correction = (
            nn.Parameter(torch.empty(E + spec.identity, dtype=torch.float32))
            if spec.correction else None)
        self.router_bias = (
            nn.Parameter(torch.empty(E + spec.identity, dtype=torch.float32))
            if spec.router_bias else None)
        # without a gate branch the tensor holds the up rows only
        self.experts_gate_up = nn.Parameter(
            torch.empty(E, (2 if spec.gated else 1) * ff, width,
                        dtype=dtype))
        self.experts_down = nn.Parameter(
            torch.empty(E, width, ff, dtype=dtype))
        self.shared = None
        self.shared_gate = None
        if spec.shared_ff:
            self.shared = GatedMLP(width, spec.shared_ff, spec.act,
                                   spec.shared_limit, dtype, spec.gated)
            if spec.shared_gate:
                self.shared_gate = nn.Parameter(
                    torch.empty(1, width, dtype=dtype))
        self._fused_in = None

    def _apply(self, fn, *a, **kw):
        # the fused input weight is a plain tensor rebuilt after a move
        self._fused_in = None
        return super()._apply(fn, *a, **kw)

    def fused_in(self) -> torch.Tensor:
        """The shared expert's gate | up | scalar-gate rows as one weight;
        the parts become views of it. Zero rows fill it up to a multiple of
        64: the odd row count a scalar gate leaves behind would cost the
        product its fast tiles and every reader its vector loads."""
        w = self._fused_in
        if w is None:
            parts = self.in_params()
            pad = -sum(p.shape[0] for p in parts) % 64
            w = torch.cat([p.data for p in parts]
                          + [parts[0].data.new_zeros(pad, parts[0].shape[1])],
                          dim=0).contiguous()
            off = 0
            for p in parts:
                p.data = w[off:off + p.shape[0]]
                off += p.shape[0]
            self._fused_in = w
        return w

    def in_params(self):
        """Parameters the caller may fold into a fused projection of the
        layer input: shared gate|up, then the shared expert's scalar
        gate."""
        if self.shared is None:
            return []
        if self.shared_gate is None:
            return [self.shared.gate_up]
        return [self.shared.gate_up, self.shared_gate]

    # up to this many rows the experts run as one grouped kernel pair whose
    # plan stays on the device; larger batches run one GEMM pair per expert
    # over the sorted rows and need the per-expert counts on the host
    GROUPED_MAX_ROWS = 128

    def load_table(self, t: torch.Tensor) -> None:
        if tuple(t.shape) != tuple(self.table.shape):
            raise ValueError(f"expert table: checkpoint shape "
                             f"{tuple(t.shape)} != {tuple(self.table.shape)}")
        if t.is_floating_point() or int(t.min()) < 0 \
                or int(t.max()) >= self.spec.experts:
            raise ValueError("expert table: entries must name experts 0 .. "
                             f"{self.spec.experts - 1}")
        self.table.data.copy_(t.to(torch.int32))

    def _all_experts(self, x: torch.Tensor, wm: torch.Tensor,
                     shared_y: Optional[torch.Tensor] = None,
                     shared_gate: Optional[torch.Tensor] = None
                     ) -> torch.Tensor:
        """Every expert over every row as batched GEMMs, without a host
        read, for what the grouped kernels do not cover (float32, odd
        widths); exact because the experts have no
        biases: a zero-weighted input (or output) contributes exactly 0.
        wm fp32 [T, router outputs]: the routing weights, zero where an
        output was not chosen. With the weight on the experts' outputs, the
        weighted sum, the identity outputs and the gated shared expert
        (shared_y [T, W], shared_gate [T, 1] pre-sigmoid, None = joins
        unscaled) are one kernel."""
        sp = self.spec
        T, E, ff = x.shape[0], sp.experts, sp.ff
        if sp.weight_on_input:
            w_id = (wm[:, E:].sum(dim=1, keepdim=True) if sp.identity
                    else None)
            we = wm[:, :E].t().unsqueeze(-1)            # [E, T, 1]
            xe = (x.float().unsqueeze(0) * we).to(x.dtype)
        else:
            xe = x.unsqueeze(0).expand(E, T, x.shape[1])
        gu = torch.bmm(xe, _right(self.experts_gate_up))
        act = self._act(gu.view(E * T, gu.shape[2]))
        y = torch.bmm(act.view(E, T, ff), _right(self.experts_down))
        if not sp.weight_on_input:
            return ops.moe_combine(y, wm, x, E, shared_y, shared_gate)
        y = y.float().sum(dim=0)
        if w_id is not None:
            y += x.float() * w_id
        if shared_y is not None:
            y += (shared_y.float() * torch.sigmoid(shared_gate.float())
                  if shared_gate is not None else shared_y.float())
        return y

    def _act(self, gu: torch.Tensor) -> torch.Tensor:
        """[n, gate | up rows] -> activation [n, ff]."""
        sp = self.spec
        if sp.gated:
            return ops.gated_act(gu[:, :sp.ff], gu[:, sp.ff:], sp.act,
                                 sp.limit)
        return ops.gated_act(gu, None, sp.act, sp.limit, out=gu)

    def _expert(self, e: int, xe: torch.Tensor) -> torch.Tensor:
        if e >= self.spec.experts:      # identity expert
            return xe
        act = self._act(gemm_policy.linear(xe, self.experts_gate_up[e]))
        return gemm_policy.linear(act, self.experts_down[e])

    @staticmethod
    def _gemm_rows(c: int) -> int:
        """Rows of the product that runs an expert's c rows. The vendor
        library looks for a kernel anew for every row count it has not met
        (about 0.1 ms of host time, more than the product takes), so the
        counts of large batches are rounded up to a few values."""
        step = 128 if c <= 1024 else 256
        return -(-c // step) * step

    @torch.no_grad()
    def _sorted_experts(self, x: torch.Tensor,
                        plan: ExpertPlan) -> torch.Tensor:
        """Sorted entries' outputs [T * top, W] (identity entries, which
        sort last, are left unwritten): one gather, one GEMM pair per
        expert over its slice, one activation over all slices."""
        E = self.spec.experts
        counts = plan.host_counts()[:E]
        n = sum(counts)
        # an expert's product may run past its rows into those of later
        # experts (or the spare rows at the end), which come after it
        spare = 256

        def buf(cols: int) -> torch.Tensor:
            return torch.empty((plan.rows.numel() + spare, cols),
                               dtype=x.dtype, device=x.device)

        def products(src, weight, dst) -> None:
            at = 0
            for e, c in enumerate(counts):
                if c:
                    m = self._gemm_rows(c) if x.is_cuda else c
                    m = min(m, dst.shape[0] - at)
                    torch.mm(src[at:at + m], weight[e].t(),
                             out=dst[at:at + m])
                at += c

        xs = buf(x.shape[1])
        torch.index_select(x, 0, plan.rows[:n], out=xs[:n])
        gu = buf(self.experts_gate_up.shape[1])
        products(xs, self.experts_gate_up, gu)
        act = self._act(gu)
        ys = buf(x.shape[1])
        products(act, self.experts_down, ys)
        # without the spare rows
        ys = ys[:plan.rows.numel()]
        return ys

    def _grouped_fits(self, x: torch.Tensor) -> bool:
        return (ops.experts_grouped_fits(x, self.experts_gate_up,
                                         self.experts_down)
                and not (self.spec.weight_on_input and self.spec.identity))

    def _grouped(self, x: torch.Tensor, plan: ExpertPlan,
                 w_in: Optional[torch.Tensor]) -> torch.Tensor:
        sp = self.spec
        return ops.experts_grouped(
            x, self.experts_gate_up, self.experts_down, plan.offs,
            plan.rows, sp.act, sp.limit, sp.gated, w_in)

    def _routed(self, x: torch.Tensor, plan: ExpertPlan,
                shared_y: Optional[torch.Tensor],
                shared_gate: Optional[torch.Tensor],
                small: Optional[bool]) -> torch.Tensor:
        """Weighted sum of the planned experts (+ shared expert), fp32."""
        sp = self.spec
        if small is None:
            small = x.shape[0] <= self.GROUPED_MAX_ROWS
        if small and self._grouped_fits(x):
            if sp.weight_on_input:
                w_in = torch.empty(plan.pos.shape, dtype=torch.float32,
                                   device=x.device).scatter_(
                    0, plan.pos.long(), plan.weights.view(-1))
                ys = self._grouped(x, plan, w_in)
                return ops.experts_sum(ys, plan.pos, plan.top, None, 1.0,
                                       None, sp.experts, x, shared_y,
                                       shared_gate)
            ys = self._grouped(x, plan, None)
        elif small:
            return self._all_experts(x, plan.dense(sp.experts + sp.identity),
                                     shared_y, shared_gate)
        else:
            ys = self._sorted_experts(x, plan)
        return ops.experts_sum(ys, plan.pos, plan.top, plan.weights,
                               plan.weight, plan.sel, sp.experts, x,
                               shared_y, shared_gate)

    def forward_from_proj(self, x: torch.Tensor,
                          proj: Optional[torch.Tensor],
                          dense: Optional[bool] = None,
                          plan: Optional[ExpertPlan] = None
                          ) -> torch.Tensor:
        """x: layer input [T, width]; proj: the shared expert's fused
        projection [T, shared in-rows (+ 1 with a scalar gate)], further
        columns unused (None without a shared expert).
        dense=True insists on a path without a host read (what a captured
        decode step needs), None picks by batch size. plan: the step's
        routed rows, for table-routed layers. Returns fp32 [T, width]:
        several experts' outputs are summed in fp32."""
        sp = self.spec
        T = x.shape[0]
        y = gate = None
        if self.shared is not None:
            rows = self.shared.in_rows
            y = self.shared.forward_from_proj(proj[:, :rows])
            if self.shared_gate is not None:
                gate = proj[:, rows:rows + 1]
        if sp.score == "table":
            if plan is None:
                raise ValueError("table-routed experts need the step's plan")
            return self._routed(x, plan, y, gate, dense)
        # one kernel: logits, scores, choice, weights, dense weight matrix
        weights, sel, wm = ops.moe_route(
            x, self.router, sp.top, sp.score, sp.renormalize,
            self.correction, sp.route_scale, sp.renorm_eps,
            self.router_bias)
        n_out = sp.experts + sp.identity
        small = dense if dense is not None else T <= self.GROUPED_MAX_ROWS
        if small and not self._grouped_fits(x):
            return self._all_experts(x, wm, y, gate)
        if small or not sp.weight_on_input:
            offs, rows_, pos = ops.expert_plan(sel, n_out)
            return self._routed(x, ExpertPlan(
                offs, rows_, pos, sp.top, weights=weights,
                sel=sel if sp.identity else None), y, gate, small)
        out = torch.zeros(x.shape, dtype=torch.float32, device=x.device)
        sparse_moe(x, weights, sel, n_out, self._expert,
                   weight_on_input=True, out=out)
        if y is not None:
            out += (y.float() * torch.sigmoid(gate.float())
                    if gate is not None else y.float())
        return out

    def forward(self, x: torch.Tensor, dense: Optional[bool] = None,
                plan: Optional[ExpertPlan] = None) -> torch.Tensor:
        proj = (gemm_policy.linear(x, self.fused_in())
                if self.shared is not None else None)
        return self.forward_from_proj(x, proj, dense, plan)


class TablePlans:
    """Plans of a stack's table-routed layers. Which rows go to which
    expert depends on the token ids alone, so one launch per (experts, top)
    pair plans every such layer at the start of a step, and the counts that
    large batches need on the host are one read per step."""

    def __init__(self, moes: List[SparseMoE]) -> None:
        self.moes = moes
        self._stacks = None

    def _groups(self):
        if self._stacks is None or any(
                t.device != self.moes[0].table.device
                for _, t, _ in self._stacks):
            by = {}
            for i, m in enumerate(self.moes):
                by.setdefault((m.spec.experts, m.spec.top), []).append(i)
            self._stacks = [
                (idx, torch.stack([self.moes[i].table.data for i in idx]),
                 experts) for (experts, _), idx in by.items()]
        return self._stacks

    def drop(self) -> None:
        """Forget the stacked tables (after weights changed)."""
        self._stacks = None

    def plan(self, token_ids: torch.Tensor,
             on_host: bool) -> List[ExpertPlan]:
        """One plan per layer; on_host reads the counts of all of them."""
        out: List[Optional[ExpertPlan]] = [None] * len(self.moes)
        for idx, tables, experts in self._groups():
            offs, rows, pos = ops.table_plan(token_ids, tables, experts)
            host = offs.tolist() if on_host else None
            top = tables.shape[2]
            for j, i in enumerate(idx):
                counts = None
                if host is not None:
                    counts = [b - a for a, b in zip(host[j], host[j][1:])]
                out[i] = ExpertPlan(offs[j], rows[j], pos[j], top,
                                    weight=1.0 / top, counts=counts)
        return out
