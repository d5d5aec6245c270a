"""Mixers that carry a fixed-size 32-bit state per request instead of keys and values: the selective scan
(with the short convolution in front of it), the generalized delta rule, a matrix memory with exponential gates, the gated
delta rule and the state-space recurrence with one decay per head (these two behind a short convolution), and lightning
attention, whose decays are constants.  Their states live in the cache manager's state slots; a request's portion that starts at position 0 starts from zero.  Every size,
constant and tensor name is a parameter.
"""
import torch

from ..registry import MIXERS
from .base import Mixer, ParamSpec, StateNeed
from .chain_norm_parts import f32_params, linear32
from .ends import EndsMixer
from .llama_parts import _linear

_SMALL = ("conv", "conv_bias", "dt_bias", "a_log", "d_skip", "a_bias", "w0", "w2", "norm")


class _StatefulMixer(Mixer):
    capturable = True

    def bind(self, tensors):
        small = f32_params({k: v for k, v in tensors.items() if k in _SMALL})
        super().bind({**tensors, **small})

    def state(self, name):
        storage, index, _ = self.caches[name]
        return storage.slots(index)


@MIXERS.register("selective_scan")
class SelectiveScanMixer(_StatefulMixer):
    """in -> [x | z]; x through a causal convolution (bias, silu); [dt | B | C] = W_x x; dt = softplus(W_dt dt + b);
    S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n with A = -exp(A_log); y = S C + D x; (y * silu(z)) -> out.
    params: inner, state, dt_rank, conv (taps).  Tensors under the prefix: in, conv, conv.b, x, dt, dt.b, A_log, D, o.
    Keeps per request: the convolution's last taps-1 inputs and S, both 32-bit."""

    def param_specs(self):
        H, p, pre = self.ctx.hidden_size, self.params, self.prefix
        C, N, R, K = p["inner"], p["state"], p["dt_rank"], p["conv"]
        return [ParamSpec("w_in", ((pre + "in", (2 * C, H)),)),
                ParamSpec("conv", ((pre + "conv", (C, K)),)),
                ParamSpec("conv_bias", ((pre + "conv.b", (C,)),), role="vector"),
                ParamSpec("w_x", ((pre + "x", (R + 2 * N, C)),)),
                ParamSpec("w_dt", ((pre + "dt", (C, R)),)),
                ParamSpec("dt_bias", ((pre + "dt.b", (C,)),), role="vector"),
                ParamSpec("a_log", ((pre + "A_log", (C, N)),)),
                ParamSpec("d_skip", ((pre + "D", (C,)),), role="vector"),
                ParamSpec("w_o", ((pre + "o", (H, C)),))]

    def cache_needs(self):
        p = self.params
        needs = {"scan": StateNeed((p["inner"], p["state"]), torch.float32)}
        if p["conv"] > 1:
            needs["conv"] = StateNeed((p["conv"] - 1, p["inner"]), torch.float32)
        return needs

    def flops(self, rows, attended=0):
        p = self.params
        return super().flops(rows) + rows * p["inner"] * (6.0 * p["state"] + 2.0 * p["conv"])

    def forward(self, step, h):
        ops, p, w = self.ctx.ops, self.params, self.w
        C, N, R, K = p["inner"], p["state"], p["dt_rank"], p["conv"]
        xz = linear32(self.ctx, step, h, w["w_in"], "scan_xz")
        conv_state = self.state("conv") if K > 1 else None
        x = step.ws("scan_x", (step.rows, C))
        single = step.max_run == 1      # every sequence runs one row: the convolution leaves the new state itself
        ops.short_conv(xz, w["conv"], x, step, conv_state, bias_out=w["conv_bias"], activation="silu", update_state=single)
        if not single:
            ops.short_conv_state(xz, conv_state, step, K)
        # the step size's low-rank input feeds a product (compute dtype); B and C enter the recurrence (32-bit)
        low = _linear(self.ctx, step, x, w["w_x"][:R], "scan_dt_low")
        bc = linear32(self.ctx, step, x, w["w_x"][R:], "scan_bc")
        dt = linear32(self.ctx, step, low, w["w_dt"], "scan_dt")
        y = step.ws("scan_y", (step.rows, C))
        # runs of some length: step sizes and gates made ahead; long runs: walked in pieces, all pieces at once
        carry = None
        if step.max_run >= 4 * ops.SCAN_PIECE:
            carry = step.flat("scan_carry", ops.selective_scan_carry_floats(max(step.rows, step.limits.max_tokens), step.limits.max_seqs, C, N))
        ops.selective_scan(x, dt, w["dt_bias"], bc, 0, N, w["a_log"], w["d_skip"], xz[:, C:], y, self.state("scan"), step,
                           prepare=step.max_run >= 16, carry=carry)
        return linear32(self.ctx, step, y, w["w_o"], "scan_out")


@MIXERS.register("general_delta")
class GeneralDeltaMixer(_StatefulMixer):
    """The generalized delta rule.  r, k, v, g, a (with a bias) and the first step of the decay's projection are
    one fused product; per head and key channel the decay is w = exp(-exp(-1/2) sigmoid(W_w2 tanh(W_w1 h) + w0)) and
    the removal rate a = sigmoid(W_a h + b); with u = k / sqrt(|k|^2 + 1e-6):
    S <- diag(w) S - (a u)(u^T S) + k v^T, o = S^T r; every head's o is divided by its root mean square, times a
    weight over all heads, times sigmoid(g), then the output projection.
    params: heads, dim, eps, rank (of the decay's projection; 0: as the checkpoint has it).
    Tensors under the prefix: r, k, v, g, a, a.b, w1, w2, w0, norm, o.  Keeps S [heads, dim, dim] per request."""

    def param_specs(self):
        H, p, pre = self.ctx.hidden_size, self.params, self.prefix
        D, R = p["heads"] * p["dim"], p.get("rank") or -1
        return [ParamSpec("w_proj", tuple((pre + n, (D, H)) for n in ("r", "k", "v", "g", "a")) + ((pre + "w1", (R, H)),)),
                ParamSpec("a_bias", ((pre + "a.b", (D,)),), role="vector"),
                ParamSpec("w2", ((pre + "w2", (D, R)),)),
                ParamSpec("w0", ((pre + "w0", (D,)),), role="vector"),
                ParamSpec("norm", ((pre + "norm", (D,)),), role="vector"),
                ParamSpec("w_o", ((pre + "o", (H, D)),))]

    def bind(self, tensors):
        super().bind(tensors)
        D = self.params["heads"] * self.params["dim"]
        self.rank = self.w["w2"].shape[1]
        self.w["w2"] = self.w["w2"].t().contiguous()      # [rank, heads*dim]: the kernel's lanes read neighbours
        if self.w["w_proj"].shape[0] != 5 * D + self.rank:
            raise ValueError(f"general_delta {self.prefix!r}: the two steps of the decay's projection do not agree on their rank "
                             f"({self.w['w_proj'].shape[0] - 5 * D} and {self.rank})")

    def cache_needs(self):
        p = self.params
        return {"delta": StateNeed((p["heads"], p["dim"], p["dim"]), torch.float32)}

    def flops(self, rows, attended=0):
        p = self.params
        return super().flops(rows) + rows * p["heads"] * 8.0 * p["dim"] * p["dim"]

    def forward(self, step, h):
        ops, p, w = self.ctx.ops, self.params, self.w
        heads, d = p["heads"], p["dim"]
        D, T = heads * d, step.rows
        proj = linear32(self.ctx, step, h, w["w_proj"], "delta_proj")
        r, k, v, g, a = (proj[:, i * D:(i + 1) * D] for i in range(5))
        low = proj[:, 5 * D:]
        decay, au, u = (step.ws(n, (T, D), torch.float32) for n in ("delta_w", "delta_au", "delta_u"))
        ops.delta_prepare(k, a, w["a_bias"], low, w["w2"], w["w0"], decay, au, u, heads, d, T)
        o = step.ws("delta_o", (T, D), torch.float32)
        ops.delta_scan(r, k, v, decay, au, u, o, self.state("delta"), step, heads, d, d)
        gated = step.ws("delta_gated", (T, D))
        ops.head_norm_gate(o, g, w["norm"], gated, heads, d, p["eps"])
        return linear32(self.ctx, step, gated, w["w_o"], "delta_out")


@MIXERS.register("matrix_memory")
class MatrixMemoryMixer(_StatefulMixer):
    """A matrix memory with exponential gates (the mLSTM cell).  q, k, v, the output gate g and one input and one forget
    gate per head are one fused product; q is scaled by dim^(-1/2); li = cap tanh((W_i h + b_i) / cap),
    lf = logsigmoid(cap tanh((W_f h + b_f) / cap)); m' = max(lf + m, li), S' = exp(lf + m - m') S + exp(li - m') k v^T, n'
    likewise with k alone, o = S'^T q / (max(|n' . q|, exp(-m')) + 1e-6); every head's o is divided by its root mean
    square, times a weight over all heads, times sigmoid(g), then the output projection.  S, n and m start at 0.
    params: heads, dim, vdim, gate_cap, eps.  Tensors under the prefix: q, k, v, g, i, i.b, f, f.b, norm, o.
    Keeps S [heads, dim, vdim], n [heads, dim] and m [heads] per request, 32-bit."""

    def param_specs(self):
        H, p, pre = self.ctx.hidden_size, self.params, self.prefix
        heads, d, dv = p["heads"], p["dim"], p["vdim"]
        sizes = (("q", heads * d), ("k", heads * d), ("v", heads * dv), ("g", heads * dv), ("i", heads), ("f", heads))
        return [ParamSpec("w_proj", tuple((pre + n, (c, H)) for n, c in sizes)),
                ParamSpec("in_bias", ((pre + "i.b", (heads,)),), role="vector"),
                ParamSpec("keep_bias", ((pre + "f.b", (heads,)),), role="vector"),
                ParamSpec("norm", ((pre + "norm", (heads * dv,)),), role="vector"),
                ParamSpec("w_o", ((pre + "o", (H, heads * dv)),))]

    def bind(self, tensors):
        w = tensors["w_proj"]
        extra = -w.shape[0] % 16      # the few-row products take widths that are multiples of 16
        if extra:
            w = torch.cat([w, torch.zeros(extra, w.shape[1], dtype=w.dtype, device=w.device)], 0)
        small = f32_params({k: tensors[k] for k in ("in_bias", "keep_bias", "norm")})
        Mixer.bind(self, {**tensors, **small, "w_proj": w})

    def cache_needs(self):
        p = self.params
        return {"memory": StateNeed((p["heads"], p["dim"], p["vdim"]), torch.float32),
                "normalizer": StateNeed((p["heads"], p["dim"]), torch.float32),
                "maximum": StateNeed((p["heads"],), torch.float32)}

    def flops(self, rows, attended=0):
        p = self.params
        return super().flops(rows) + rows * p["heads"] * (4.0 * p["dim"] * p["vdim"] + 4.0 * p["dim"])

    def forward(self, step, h):
        ops, p, w = self.ctx.ops, self.params, self.w
        heads, d, dv = p["heads"], p["dim"], p["vdim"]
        T = step.rows
        proj = linear32(self.ctx, step, h, w["w_proj"], "memory_proj")
        at = [0, heads * d, 2 * heads * d, 2 * heads * d + heads * dv, 2 * heads * (d + dv), 2 * heads * (d + dv) + heads]
        q, k, v, g, gi, gf = (proj[:, lo:] for lo in at)
        coef = step.ws("memory_factors", (T, 4 * heads), torch.float32)
        seqs = max(step.seqs, step.limits.max_seqs if step.limits is not None else step.seqs)
        n_new = step.flat("memory_normalizer", seqs * heads * d)
        o = step.ws("memory_o", (T, heads * dv), torch.float32)
        ops.mlstm_scan(q, k, v, gi, gf, w["in_bias"], w["keep_bias"], p["gate_cap"], float(d) ** -0.5, coef, n_new, o,
                       self.state("memory"), self.state("normalizer"), self.state("maximum"), step, heads, d, dv)
        gated = step.ws("memory_gated", (T, heads * dv))
        ops.head_norm_gate(o, g, w["norm"], gated, heads, dv, p["eps"])
        return linear32(self.ctx, step, gated, w["w_o"], "memory_out", keep_partial=True)      # the stream's next norm adds the slices


class _MatrixStateMixer(EndsMixer):
    """A matrix state per head with one decay per head (ops.gated_state).  Keeps it per request, 32-bit."""

    capturable = True

    def state(self, name):
        storage, index, _ = self.caches[name]
        return storage.slots(index)


class _ConvStateMixer(_MatrixStateMixer):
    """A short convolution (silu) over some of the projected channels, then a matrix state per head with one decay per head
    and token.  Keeps per request: the state and the convolution's last taps-1 inputs, both 32-bit."""

    def needs(self, heads, dk, dv, taps, channels):
        needs = {"state": StateNeed((heads, dk, dv), torch.float32)}
        if taps > 1:
            needs["conv"] = StateNeed((taps - 1, channels), torch.float32)
        return needs

    def convolved(self, step, x, bias=None):
        """The convolution of the columns of x (as many as it has channels), 32-bit; its new inputs left in the slot."""
        ops, weight = self.ctx.ops, self.w["conv"]
        C, taps = weight.shape
        mixed = step.ws(self.ends_name + "_conv", (step.rows, C), torch.float32)
        state = self.state("conv") if taps > 1 else None
        single = step.max_run == 1      # every sequence runs one row: the convolution leaves the new state itself
        ops.short_conv(x, weight, mixed, step, state, bias_out=bias, activation="silu", update_state=single)
        if not single:
            ops.short_conv_state(x, state, step, taps)
        return mixed

    def carry(self, step, heads, dk, dv, delta):
        """Scratch for walking long runs in pieces, sized for the engine's largest step; None for steps of short runs."""
        ops = self.ctx.ops
        if step.max_run < 4 * ops.gated_state_piece(dk):
            return None
        lim = step.limits
        rows, seqs = max(step.rows, lim.max_tokens if lim else 0), max(step.seqs, lim.max_seqs if lim else 0)
        return step.flat("gated_state_carry", ops.gated_state_carry_floats(rows, seqs, heads, dk, dv, delta))


@MIXERS.register("gated_delta")
class GatedDeltaMixer(_ConvStateMixer):
    """The gated delta rule.  q, k (kv_heads heads of dim) and v (heads of vdim) pass a causal convolution per channel and
    silu; q and k become unit vectors per head (x / sqrt(|x|^2 + 1e-6)), q times dim^(-1/2); head h reads q and k head
    h / (heads / kv_heads).  beta = sigmoid(W_b h), g = exp(-exp(A_log) softplus(W_a h + dt_bias)), one each per head;
    S <- g S, u = beta (v - S^T k), S <- S + k u^T, o = S^T q; every head's o is divided by its root mean square, times one
    weight of the head's size that all heads share, times silu(W_g h), then the output projection.
    params: heads, kv_heads, dim, vdim, conv (taps), eps, out_factor (on the output, default 1).
    Tensors under the prefix: q, k, v (each + ".conv"), g, b, a, A_log, dt_bias, norm, o."""

    ends_name = "gated_delta"

    def __init__(self, params, prefix, ctx):
        super().__init__(params, prefix, ctx)
        p = params
        self.nh, self.nkv, self.d, self.dv = p["heads"], p["kv_heads"], p["dim"], p["vdim"]
        if self.nkv <= 0 or self.nh % self.nkv:
            raise ValueError(f"gated_delta {prefix!r}: heads {self.nh} is not a multiple of kv_heads {self.nkv}")
        self.qk = self.nkv * self.d
        self.channels = 2 * self.qk + self.nh * self.dv

    def in_sources(self):
        H, pre, nv = self.ctx.hidden_size, self.prefix, self.nh * self.dv
        return tuple((pre + n, (c, H)) for n, c in (("q", self.qk), ("k", self.qk), ("v", nv), ("g", nv), ("b", self.nh), ("a", self.nh)))

    def out_source(self):
        return (self.prefix + "o", (self.ctx.hidden_size, self.nh * self.dv))

    def own_specs(self):
        pre, K = self.prefix, self.params["conv"]
        return [ParamSpec("conv", tuple((pre + n + ".conv", (c, K)) for n, c in (("q", self.qk), ("k", self.qk), ("v", self.nh * self.dv)))),
                ParamSpec("a_log", ((pre + "A_log", (self.nh,)),), role="bias"),
                ParamSpec("dt_bias", ((pre + "dt_bias", (self.nh,)),), role="bias"),
                ParamSpec("norm", ((pre + "norm", (self.dv,)),), role="vector")]

    def bind(self, tensors):
        super().bind(tensors)
        # the shared weight once per head, the output's factor in it
        self.w["norm"] = (self.w["norm"].repeat(self.nh) * float(self.params.get("out_factor", 1.0))).contiguous()

    def cache_needs(self):
        return self.needs(self.nh, self.d, self.dv, self.params["conv"], self.channels)

    def flops(self, rows, attended=0):
        return super().flops(rows) + rows * self.nh * 7.0 * self.d * self.dv + 2.0 * rows * self.channels * self.params["conv"]

    def between(self, step, h, proj, out):
        ops, p, w = self.ctx.ops, self.params, self.w
        nh, d, dv = self.nh, self.d, self.dv
        mixed = self.convolved(step, proj)
        q, k, v = mixed, mixed[:, self.qk:], mixed[:, 2 * self.qk:]
        g, b, a = (proj[:, at:] for at in (self.channels, self.channels + nh * dv, self.channels + nh * dv + nh))
        o = step.ws("gated_delta_o", (step.rows, nh * dv), torch.float32)
        ops.gated_state(q, k, v, a, w["dt_bias"], w["a_log"], o, self.state("state"), step, nh, self.nkv, d, dv, b=b,
                        carry=self.carry(step, nh, d, dv, True))
        ops.head_norm_gate(o, g, w["norm"], out, nh, dv, p["eps"], activation="silu")


@MIXERS.register("state_space_duality")
class StateSpaceMixer(_ConvStateMixer):
    """The state-space recurrence with one decay per head (Mamba-2's).  in -> [z | x | B | C | dt]; x, B and C pass a causal
    convolution per channel (bias, silu); dt = softplus(dt + dt_bias); head h reads B and C of group h / (heads / groups);
    S <- exp(-exp(A_log) dt) S + dt B x^T, y = S^T C + D x; y * silu(z), divided by the root mean square of each of
    norm_groups equal parts, times a weight, then the output projection.
    params: heads, vdim, state, groups, norm_groups, conv (taps), eps, out_factor (on the output, default 1).
    Tensors under the prefix: in, conv, conv.b, A_log, dt_bias, D, norm, o."""

    ends_name = "state_space"

    def __init__(self, params, prefix, ctx):
        super().__init__(params, prefix, ctx)
        p = params
        self.nh, self.dv, self.N, self.groups, self.norm_groups = p["heads"], p["vdim"], p["state"], p["groups"], p["norm_groups"]
        self.inner = self.nh * self.dv
        self.channels = self.inner + 2 * self.groups * self.N
        if self.nh % self.groups or self.inner % self.norm_groups:
            raise ValueError(f"state_space_duality {prefix!r}: {self.nh} heads in {self.groups} groups, {self.inner} channels in "
                             f"{self.norm_groups} parts do not come out even")

    def in_sources(self):
        return ((self.prefix + "in", (self.inner + self.channels + self.nh, self.ctx.hidden_size)),)

    def out_source(self):
        return (self.prefix + "o", (self.ctx.hidden_size, self.inner))

    def own_specs(self):
        pre = self.prefix
        return [ParamSpec("conv", ((pre + "conv", (self.channels, self.params["conv"])),)),
                ParamSpec("conv_bias", ((pre + "conv.b", (self.channels,)),), role="bias"),
                ParamSpec("a_log", ((pre + "A_log", (self.nh,)),), role="bias"),
                ParamSpec("dt_bias", ((pre + "dt_bias", (self.nh,)),), role="bias"),
                ParamSpec("d_skip", ((pre + "D", (self.nh,)),), role="vector"),
                ParamSpec("norm", ((pre + "norm", (self.inner,)),), role="vector")]

    def bind(self, tensors):
        super().bind(tensors)
        self.w["norm"] = (self.w["norm"] * float(self.params.get("out_factor", 1.0))).contiguous()

    def cache_needs(self):
        return self.needs(self.nh, self.N, self.dv, self.params["conv"], self.channels)

    def flops(self, rows, attended=0):
        return super().flops(rows) + rows * self.nh * 5.0 * self.N * self.dv + 2.0 * rows * self.channels * self.params["conv"]

    def between(self, step, h, proj, out):
        ops, p, w = self.ctx.ops, self.params, self.w
        inner, GN = self.inner, self.groups * self.N
        mixed = self.convolved(step, proj[:, inner:], bias=w["conv_bias"])
        y = step.ws("state_space_y", (step.rows, inner), torch.float32)
        ops.gated_state(mixed[:, inner + GN:], mixed[:, inner:], mixed, proj[:, inner + self.channels:], w["dt_bias"], w["a_log"], y,
                        self.state("state"), step, self.nh, self.groups, self.N, self.dv, d_skip=w["d_skip"],
                        carry=self.carry(step, self.nh, self.N, self.dv, False))
        ops.group_norm_gate(y, proj, w["norm"], out, self.norm_groups, inner // self.norm_groups, p["eps"])


@MIXERS.register("lightning_attention")
class LightningAttention(_MatrixStateMixer):
    """Linear attention with a constant decay per head.  q = silu(W_q h), k = silu(W_k h) (heads of dim), v = silu(W_v h) (heads
    of vdim); S <- decay_h S + k v^T, o = S^T q; all heads' o side by side are divided by their root mean square together, times
    a weight, times sigmoid(W_g h), then the output projection.
    params: heads, dim, vdim, decay (a number per head), eps, out_factor (on the output, default 1).
    Tensors under the prefix: q, k, v, g, norm, o."""

    ends_name = "lightning"

    def __init__(self, params, prefix, ctx):
        super().__init__(params, prefix, ctx)
        self.nh, self.d, self.dv = params["heads"], params["dim"], params["vdim"]
        if len(params["decay"]) != self.nh:
            raise ValueError(f"lightning_attention {prefix!r}: {len(params['decay'])} decays for {self.nh} heads")

    def in_sources(self):
        H, pre, nk, nv = self.ctx.hidden_size, self.prefix, self.nh * self.d, self.nh * self.dv
        return tuple((pre + n, (c, H)) for n, c in (("q", nk), ("k", nk), ("v", nv), ("g", nv)))

    def out_source(self):
        return (self.prefix + "o", (self.ctx.hidden_size, self.nh * self.dv))

    def own_specs(self):
        return [ParamSpec("norm", ((self.prefix + "norm", (self.nh * self.dv,)),), role="vector")]

    def bind(self, tensors):
        super().bind(tensors)
        self.w["norm"] = (self.w["norm"] * float(self.params.get("out_factor", 1.0))).contiguous()
        device = self.w["norm"].device
        self.w["decay"] = torch.tensor(self.params["decay"], dtype=torch.float32, device=device)
        if self.ctx.ops is not None:
            self.w["powers"] = self.ctx.ops.lightning_powers(self.params["decay"], self.ctx.ops.lightning_piece(self.d), device)

    def cache_needs(self):
        return {"state": StateNeed((self.nh, self.d, self.dv), torch.float32)}

    def carry(self, step):
        """Scratch for runs longer than a piece, sized for the engine's largest step."""
        ops, lim = self.ctx.ops, step.limits
        if step.max_run <= ops.lightning_piece(self.d):
            return None
        rows, seqs = max(step.rows, lim.max_tokens if lim else 0), max(step.seqs, lim.max_seqs if lim else 0)
        return step.flat("lightning_carry", ops.lightning_carry_floats(rows, seqs, self.nh, self.d, self.dv))

    def flops(self, rows, attended=0):
        return super().flops(rows) + rows * self.nh * 5.0 * self.d * self.dv

    def between(self, step, h, proj, out):
        ops, w = self.ctx.ops, self.w
        nh, d, dv = self.nh, self.d, self.dv
        q, k, v, g = (proj[:, at:] for at in (0, nh * d, 2 * nh * d, 2 * nh * d + nh * dv))
        o = step.ws("lightning_o", (step.rows, nh * dv), torch.float32)
        if step.max_run >= ops.LIGHTNING_MIN_RUN:      # runs of rows: products on the matrix cores, chunk by chunk
            ops.lightning(q, k, v, w["powers"], o, self.state("state"), step, nh, d, dv, silu_in=True, carry=self.carry(step))
        else:
            ops.gated_state(q, k, v, None, None, None, o, self.state("state"), step, nh, nh, d, dv, decay=w["decay"], silu_in=True)
        ops.group_norm_gate(o, g, w["norm"], out, 1, nh * dv, self.params["eps"], after=True)
