"""Linear attention with a decay per head, or per key channel and token (config/schema.py: LinearAttentionSpec): a recurrent mixer whose
per-request state has a fixed size, one matrix S [dim, vdim] per head in fp32 (kept column by column, [vdim, dim]) in the
cache manager's state slots. Nothing is paged and nothing grows with the context.

A step is
  1. one product with the stacked weight [W_q | W_k | W_v | W_g] (and, where the token chooses its decays, the narrow W_down
     of their input),
  2. the recurrence over each request's rows in order, with the activation, the rotation, k's constant and the second half
     of the decays' input inside
     (``ops.linear_attention``; its read-out comes back raw, in fp32): row by row for steps of few rows per request, in
     chunks of 64 rows as fp32 matrix products for portions of prompts,
  3. the norm of every head (``ops.heads_finish``, the kernel that ends attention heads too) or of the whole row
     (``ops.gated_group_norm``) and the gate,
  4. the output product.
"""
from __future__ import annotations

import torch

from ..cache.manager import StateSpec
from ..config.schema import LinearAttentionSpec
from ..kernels import ops
from ..weights.loader import WeightSpec
from .base import BuildContext, Part, pad_rows, register_part


class LinearStepPlanner:
    """The step's rows in chunks, once per step for all such layers: for steps with a portion long enough for the chunked
    form; steps of few rows per request (and steps of fixed size, whose requests have one row each) get an empty plan."""

    key = ("linear_attention", ops.LINEAR_CHUNK)

    def plan(self, batch):
        from ..engine.step import StepPlan
        if batch.padded or max((s.n for s in batch.segments), default=0) < ops.LINEAR_CHUNK_FROM:
            return StepPlan({"requests": [], "chunks": []})
        requests, chunks = ops.linear_chunk_plan(batch.segments)
        return StepPlan({"requests": requests, "chunks": chunks})


class LinearAttention(Part):
    def __init__(self, spec: LinearAttentionSpec, prefix: str, build: BuildContext, positions):
        if spec.decay_per not in ("head", "channel"):
            raise ValueError(f"{prefix}: a decay per '{spec.decay_per}' is not built ('head' and 'channel' are)")
        self.channel = spec.decay_per == "channel"
        if len(spec.decay) != (0 if self.channel else spec.heads):
            raise ValueError(f"{prefix}: {len(spec.decay)} fixed decays for {spec.heads} heads with a decay per {spec.decay_per}")
        if self.channel and (not spec.tau > 0 or spec.decay_rank == 0 or spec.position is not None):
            raise ValueError(f"{prefix}: a decay per key channel takes its input through a narrow middle ({spec.decay_rank}), with a "
                             f"positive tau ({spec.tau}) and without a rotation")
        if spec.activation not in (None, "silu"):
            raise ValueError(f"{prefix}: activation '{spec.activation}' in front of the recurrence (silu is built)")
        if spec.norm not in ("head", "head_gain", "whole"):
            raise ValueError(f"{prefix}: norm '{spec.norm}' of the read-out ('head', 'head_gain' and 'whole' are built)")
        if spec.gate_fn not in ops.HEAD_GATES:
            raise ValueError(f"{prefix}: gate function '{spec.gate_fn}' ({sorted(ops.HEAD_GATES)} are built)")
        self.spec = spec
        self.prefix = prefix
        self.build = build
        position = positions[spec.position] if spec.position is not None else None
        self.rot = position.rotary() if position is not None else None
        if self.rot is not None and position.pairing != "half":
            raise ValueError(f"{prefix}: rotary pairing '{position.pairing}' ('half' is built for this mixer)")
        try:
            ops.check_linear_shape(spec.heads, spec.dim, spec.vdim, self.rot[2] if self.rot else 0)
        except ops.KernelError as e:
            raise ValueError(f"{prefix}: {e}") from None
        self.qk_dim = spec.heads * spec.dim
        self.v_dim = spec.heads * spec.vdim
        self.decay_at = 2 * self.qk_dim + 2 * self.v_dim  # the stacked product's columns behind q | k | v | gate
        self.w_in = self.w_o = self.gain = self.powers = self.w_decay_up = self.b_decay = self.decay_rank = None

    def _name(self, which: str) -> str:
        return f"{self.prefix}.{getattr(self.spec.names, which)}"

    def weight_specs(self):
        d = self.build.hidden
        out = [WeightSpec(self._name("q"), (self.qk_dim, d)), WeightSpec(self._name("k"), (self.qk_dim, d)),
               WeightSpec(self._name("v"), (self.v_dim, d)), WeightSpec(self._name("gate"), (self.v_dim, d)),
               WeightSpec(self._name("o"), (d, self.v_dim))]
        if self.spec.norm != "head":
            out.append(WeightSpec(self._name("norm"), (self.v_dim if self.spec.norm == "whole" else self.spec.vdim,), init="gain"))
        if self.channel:
            r = self.spec.decay_rank
            out += [WeightSpec(self._name("decay_down"), (r, d)), WeightSpec(self._name("decay_up"), (self.qk_dim, r)),
                    WeightSpec(self._name("decay_bias"), (self.qk_dim,), init="bias")]
        return out

    def load(self, get):
        stack = [get(self._name(n)) for n in ("q", "k", "v", "gate") + (("decay_down",) if self.channel else ())]
        if self.channel:
            up = get(self._name("decay_up"))
            self.b_decay = get(self._name("decay_bias")).float().contiguous()
            if up.shape[1] != stack[-1].shape[0]:
                raise ValueError(f"{self.prefix}: the two halves of the decay's input disagree about their middle: "
                                 f"{stack[-1].shape[0]} and {up.shape[1]}")
            self.decay_rank = up.shape[1]
            # the middle filled up with zeros, on both sides, to what the recurrence takes
            stack[-1] = pad_rows(stack[-1], ops.LINEAR_MIDDLE)
            self.w_decay_up = pad_rows(up.t().to(self.build.dtype), ops.LINEAR_MIDDLE).t().contiguous()
        dt = stack[0].dtype if all(t.dtype == stack[0].dtype for t in stack) else torch.float32
        self.w_in = pad_rows(torch.cat([t.to(dt) for t in stack], dim=0).contiguous())
        self.w_o = get(self._name("o"))
        if self.spec.norm != "head":
            self.gain = get(self._name("norm"))
        if not self.channel:
            self.powers = ops.decay_powers(self.spec.decay, self.build.device)

    def state_spec(self):
        s = self.spec
        return StateSpec((s.heads, s.vdim, s.dim), torch.float32)

    def step_planners(self):
        return [LinearStepPlanner()]

    # what a mixer beside others on the same input shares with them (parts/parallel.py)
    def input_projection(self):
        return self.w_in, None

    def output_weight(self):
        return self.w_o

    @property
    def heads_width(self):
        return self.v_dim

    def heads_rows(self, xb, step, slot):
        """The input of the output product, [rows, heads x vdim] in the run's type."""
        y = ops.gemm(xb, self.w_in, out_dtype=self.build.dtype, exact=self.build.exact)
        return self.heads_rows_from(y, step, slot)

    def heads_rows_from(self, y, step, slot, out=None, out_mul=1.0):
        """The same from the input product's result ``y`` (a view with any row stride); ``out``: where to write."""
        s = self.spec
        cos, sin, rdims = self.rot if self.rot is not None else (None, None, 0)
        plan = step.plans.get(LinearStepPlanner.key)
        requests = plan.arrays.get("requests") if plan is not None else None
        chunks = plan.arrays.get("chunks") if plan is not None else None
        o = ops.linear_attention(y, 0, self.qk_dim, 2 * self.qk_dim, self.powers, slot.state, step.row_req, step.state_slots,
                                 step.n_requests, s.heads, s.dim, s.vdim, positions=step.positions, cos=cos, sin=sin,
                                 rot_dims=rdims, silu=s.activation == "silu", k_scale=s.k_scale, requests=requests, chunks=chunks,
                                 decay_off=self.decay_at, decay_up=self.w_decay_up, decay_bias=self.b_decay,
                                 decay_rank=self.decay_rank, tau=s.tau)
        gate_at = 2 * self.qk_dim + self.v_dim
        gate = y[:, gate_at:gate_at + self.v_dim]
        if s.norm != "whole":
            return ops.heads_finish(o, s.heads, 1, s.vdim, self.build.dtype, normed=True, eps=s.eps, gain=self.gain, gate=gate,
                                    gate_fn=s.gate_fn, out=out, out_mul=out_mul)
        return ops.gated_group_norm(o, gate, self.gain, s.eps, 1, self.build.dtype, gate_fn=s.gate_fn, gate_last=True, out=out,
                                    out_mul=out_mul)

    def output(self, xb, step, slot):
        return ops.gemm(self.heads_rows(xb, step, slot), self.w_o, out_dtype=torch.float32, exact=self.build.exact)

    def forward(self, xb, residual, step, slot):
        ops.gemm(self.heads_rows(xb, step, slot), self.w_o, out=residual, epilogue=ops.EPI_ADD, exact=self.build.exact)


register_part("mixer", "linear_attention", LinearAttention, replace=True)
