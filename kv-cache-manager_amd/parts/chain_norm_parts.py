"""Parts for layers that norm a sublayer's output before adding it to the residual stream
(x += norm_out(sublayer(norm_in(x))), or x += norm_out(sublayer(x)) where the sublayers read the stream itself):
an RMS norm whose arithmetic is 32-bit throughout, the arrangements that chain such norms so that a layer boundary
is one launch, an embedding with a factor, and a gated feed-forward with a choice of activation.  Every size, constant and tensor name is a parameter.
"""
import torch

from ..registry import BLOCKS, EMBEDDINGS, FEED_FORWARDS, NORMS
from .base import Block, Embedding, FeedForward, JoinableEnds, Norm, ParamSpec
from .llama_parts import _linear


def f32_params(tensors):
    """Small tensors (norm weights, biases, per-head factors, convolution taps) as float32: widening what a
    checkpoint stores in 16 bits is exact, and the kernels that use them compute in 32-bit."""
    return {k: v.float().contiguous() for k, v in tensors.items()}


def pad_rows(t, multiple=16):
    """A matrix with zero rows appended up to a multiple (the few-row products take such widths)."""
    extra = -t.shape[0] % multiple
    if not extra:
        return t
    return torch.cat([t, torch.zeros(extra, t.shape[1], dtype=t.dtype, device=t.device)], 0)


def linear32(ctx, step, x, w, name, keep_partial=False):
    """x @ w^T as 32-bit rows for a consumer that computes in 32-bit: the product's 32-bit sums as they are, from this
    package's kernels for few rows and from the vendor library's for many (``ops.gemm`` decides, as for every product);
    no path rounds the sums, so what enters a recurrence is as exact at one row as at thousands.  Few-row products stay
    split along K with a second launch that adds the slices up: run unsplit they were slower by more than that launch
    costs (a decode step at width 2048 0.71 -> 0.80 ms, at 4096 1.25 -> 1.49 ms).  ``keep_partial``: the product may come
    back as ops.PartialSums for a consumer that adds the slices itself.  The chained norm does: rows up to 8,192 wide
    stay in registers through all its stages, and the slices are added as they are loaded (5 us a launch at width 2048;
    the form that reads a row once per stage took 27 us with slices, more than the launch it saved).  Mixers' output
    projections use it; a feed-forward's does not where another part (a routed feed-forward's sum) starts from it."""
    return _linear(ctx, step, x, w, name, keep_partial=keep_partial, dtype=torch.float32)


class BranchPair:
    """Two sublayer outputs (32-bit tensors, or the un-added slices of their last products) side by side, still to be combined as combine * (n(a) * wa + n(b) * wb)
    (n: division by the root mean square): what a mixer of two halves hands to the arrangement, which
    passes it on to the norm that adds it to the stream (one launch for all of it)."""

    def __init__(self, a, wa, b, wb, combine):
        self.a, self.wa, self.b, self.wb, self.combine = a, wa, b, wb, combine


@NORMS.register("rmsnorm_chain")
class ChainedRMSNorm(Norm):
    """out = x / sqrt(mean(x^2) + eps) * weight with every operation in 32-bit and one rounding at the end.
    ``forward`` also takes the previous sublayer's output that is still to be normed and added (``add``: what
    ``pending`` of the norm after that sublayer made), so that addition and norm are one launch.
    params: size, eps; offset: the weight is stored around it, the factor is offset + weight (default 0); factor: a constant
    on the factor, for a norm whose result is added to the stream multiplied (default 1); name: the checkpoint name of the
    weight (default prefix + "weight")."""

    capturable = True
    accepts_partial_sums = True      # ``add`` is taken as it comes (ops.NormedBranches)

    def param_specs(self):
        name = self.params.get("name", self.prefix + "weight")
        return [ParamSpec("weight", ((name, (self.params["size"],)),), role="bias" if self.params.get("offset") else "vector")]

    def bind(self, tensors):
        w = f32_params(tensors)["weight"]
        offset, factor = float(self.params.get("offset", 0.0)), float(self.params.get("factor", 1.0))
        if offset != 0.0 or factor != 1.0:
            w = ((w + offset) * factor).contiguous()
        super().bind({"weight": w})

    def pending(self, value):
        """A sublayer's output (a 32-bit tensor, ops.PartialSums, a BranchPair, or ops.StreamTerms of one plain term) as what the
        stream's next norm adds: x += n(value) * weight."""
        ops = self.ctx.ops
        if isinstance(value, ops.StreamTerms):
            value = value.only()
        if isinstance(value, BranchPair):
            return ops.NormedBranches(value.a, self.w["weight"], value.b, value.wa, value.wb, value.combine)
        return ops.NormedBranches(value, self.w["weight"])

    def forward(self, x, out, add=None, rows=None):
        ops = self.ctx.ops
        if add is not None and not isinstance(add, ops.NormedBranches):
            raise TypeError("rmsnorm_chain adds what a norm's pending() made (ops.NormedBranches)")
        ops.rmsnorm_chain(x, self.params["eps"], pending=add, weight=self.w["weight"], out=out, rows=rows)
        return out

    def read_stream(self, step, x, add=None):
        """x += what is still to be added (``add``: made by a norm's ``pending``), then the stream's rows as a sublayer
        reads them that takes the stream itself, not a normed copy: rounded to the compute dtype in the same launch, or,
        where the compute dtype is 32-bit, x itself."""
        ops = self.ctx.ops
        if add is not None and not isinstance(add, ops.NormedBranches):
            raise TypeError("rmsnorm_chain adds what a norm's pending() made (ops.NormedBranches)")
        if self.ctx.dtype == torch.float32:
            if add is not None:
                ops.rmsnorm_chain(x, self.params["eps"], pending=add)
            return x
        out = step.ws("stream_rows", (step.rows, x.shape[1]))
        ops.rmsnorm_chain(x, self.params["eps"], pending=add, out=out, plain=True)
        return out


@BLOCKS.register("sandwich_residual")
class SandwichResidual(Block):
    """x += norm_mixer_out(mixer(norm_mixer(x))); x += norm_ffn_out(ffn(norm_ffn(x))), the second half only
    where the layer has a feed-forward.  Each addition is done by the norm that reads the stream next."""

    capturable = True

    def forward(self, step, x, pending):
        p = self.parts
        buf = step.ws("normed", (step.rows, x.shape[1]))
        p["norm_mixer"].forward(x, buf, add=pending)
        pending = p["norm_mixer_out"].pending(p["mixer"].forward(step, buf))
        if "ffn" in p:
            p["norm_ffn"].forward(x, buf, add=pending)
            pending = p["norm_ffn_out"].pending(p["ffn"].forward(step, buf))
        return pending


@BLOCKS.register("output_norm_residual")
class OutputNormResidual(Block):
    """x += norm_mixer_out(mixer(x)); x += norm_ffn_out(ffn(x)), the second half only where the layer has a
    feed-forward.  No norm on the way in: the sublayers read the stream itself.  Each addition is done by the launch
    that hands the stream to its next reader."""

    capturable = True

    def forward(self, step, x, pending):
        p = self.parts
        h = p["norm_mixer_out"].read_stream(step, x, add=pending)
        pending = p["norm_mixer_out"].pending(p["mixer"].forward(step, h))
        if "ffn" in p:
            h = p["norm_ffn_out"].read_stream(step, x, add=pending)
            pending = p["norm_ffn_out"].pending(p["ffn"].forward(step, h))
        return pending


@EMBEDDINGS.register("scaled_token_embedding")
class ScaledTokenEmbedding(Embedding):
    """x = float(table[token]) * scale; with ``positions`` (a number of them) a learned vector per position is added as it is.
    params: vocab_size, scale; name: the table's checkpoint name; positions; position_name: the checkpoint name of their table."""

    capturable = True

    def param_specs(self):
        name, p, H = self.params.get("name", self.prefix + "weight"), self.params, self.ctx.hidden_size
        specs = [ParamSpec("table", ((name, (p["vocab_size"], H)),), role="table")]
        if p.get("positions"):
            specs.append(ParamSpec("pos_table", ((p.get("position_name", self.prefix + "positions"), (p["positions"], H)),), role="table"))
        return specs

    def forward(self, step, out):
        self.ctx.ops.embed_scaled(step.tokens, self.w["table"], out, self.params.get("scale", 1.0),
                                  positions=step.positions if "pos_table" in self.w else None, pos_table=self.w.get("pos_table"))
        return out

    def bytes_read(self, rows):
        return sum(rows * t.shape[1] * t.element_size() for t in self.w.values())

    def flops(self, rows, attended=0):
        return 0.0


@FEED_FORWARDS.register("gated_mlp")
class GatedFeedForward(JoinableEnds, FeedForward):
    """down(act(gate(h)) * up(h)), gate and up as one fused projection whose 32-bit sums go straight into the
    activation (steps of few rows in bfloat16 with silu or "clamped" and without biases: in the product's own epilogue).
    params: intermediate_size, activation ("relu" | "silu" | "gelu_tanh" | "gelu", or "clamped" with ``limit``: g * sigmoid(1.702 g) *
    (u + 1) with g = min(gate, limit) and u = up held within +-limit); gate, up, down: the
    checkpoint names after the prefix (defaults "gate", "up", "down"); bias: all three projections have one (the tensor's
    name + ".b"); partial_out: the last product may be handed on as un-added slices, to a norm that adds them (default: not).
    The result is 32-bit: a norm reads it.  Offers its ends (JoinableEnds)."""

    capturable = True

    def in_sources(self):
        H, I, pre, p = self.ctx.hidden_size, self.params["intermediate_size"], self.prefix, self.params
        return ((pre + p.get("gate", "gate"), (I, H)), (pre + p.get("up", "up"), (I, H)))

    def out_source(self):
        return (self.prefix + self.params.get("down", "down"), (self.ctx.hidden_size, self.params["intermediate_size"]))

    def out_bias(self):
        return self.w.get("b_down")

    def param_specs(self):
        specs = [] if self.params.get("joined") else [ParamSpec("w_gate_up", self.in_sources()), ParamSpec("w_down", (self.out_source(),))]
        if self.params.get("bias"):
            specs += [ParamSpec("b_gate_up", tuple((n + ".b", s[:1]) for n, s in self.in_sources()), role="bias"),
                      ParamSpec("b_down", ((self.out_source()[0] + ".b", (self.ctx.hidden_size,)),), role="bias")]
        return specs

    def bind(self, tensors):
        small = f32_params({k: v for k, v in tensors.items() if k.startswith("b_")})
        super().bind({**tensors, **small})

    def between(self, step, h, proj, out, row_gate=None):
        """``row_gate`` (32-bit rows, column 0): the output times sigmoid of it, one gate per row."""
        self.ctx.ops.gated_act(proj, out, self.params.get("activation", "silu"), bias=self.w.get("b_gate_up"), row_gate=row_gate,
                               limit=self.params.get("limit", 0.0))

    def forward(self, step, h):
        I, ops = self.params["intermediate_size"], self.ctx.ops
        if self.params.get("bias"):
            act = step.ws("gated_act", (step.rows, I))
            self.between(step, h, linear32(self.ctx, step, h, self.w["w_gate_up"], "gated_gate_up"), act)
            return ops.BiasedOutput(linear32(self.ctx, step, act, self.w["w_down"], "gated_out", keep_partial=True), self.w["b_down"])
        act = step.ws("gated_act", (step.rows, I))
        kind = self.params.get("activation", "silu")
        limit = self.params.get("limit", 0.0) if kind == "clamped" else 0.0
        # few rows in bfloat16 with silu or its form with limits: the product that streams gate and up rows together and applies
        # the activation in its epilogue, one launch (silu is rounded once more on the way, within the result's own rounding)
        if not (kind in ("silu", "clamped") and act.dtype == torch.bfloat16 and torch.is_tensor(h)
                and ops.gemm_swiglu(h, self.w["w_gate_up"], act, limit=limit)):
            gu = linear32(self.ctx, step, h, self.w["w_gate_up"], "gated_gate_up")
            ops.gated_act(gu, act, kind, limit=limit)
        return linear32(self.ctx, step, act, self.w["w_down"], "gated_out", keep_partial=bool(self.params.get("partial_out")))


@FEED_FORWARDS.register("plain_mlp")
class PlainFeedForward(FeedForward):
    """down(act(up(h))): a feed-forward without a gate; the first product's 32-bit sums go straight into the activation.
    params: intermediate_size, activation ("relu" | "silu" | "gelu_tanh"); up, down: the checkpoint names after the
    prefix (defaults "up", "down").  The result is 32-bit: a norm reads it."""

    capturable = True

    def param_specs(self):
        H, I, pre, p = self.ctx.hidden_size, self.params["intermediate_size"], self.prefix, self.params
        return [ParamSpec("w_up", ((pre + p.get("up", "up"), (I, H)),)),
                ParamSpec("w_down", ((pre + p.get("down", "down"), (H, I)),))]

    def forward(self, step, h):
        I, ops = self.params["intermediate_size"], self.ctx.ops
        up = linear32(self.ctx, step, h, self.w["w_up"], "plain_up", keep_partial=True)      # slices are added by the activation's launch
        act = step.ws("plain_act", (step.rows, I))
        ops.act_rows(up, act, self.params.get("activation", "gelu_tanh"))
        return linear32(self.ctx, step, act, self.w["w_down"], "plain_out", keep_partial=True)      # the stream's next norm adds the slices
