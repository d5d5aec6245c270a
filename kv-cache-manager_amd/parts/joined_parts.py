"""Parts for layers whose sublayers all read one normed copy of the stream, x <- x + sum of factor_i * sublayer_i(n(x)):

  joined_sublayers    any number of sublayers (mixers and feed-forwards) driven as one: their first products are one product,
                      their last products are one product too (their inputs side by side, their matrices side by side), so
                      that adding the sublayers up costs nothing
  parallel_residual   the arrangement; a layer boundary is one launch (the outputs added, the stream normed)
  offset_rmsnorm      an RMS norm whose weight is stored around a constant, all arithmetic in 32-bit
  embedding_again     the embedding's output added to the stream once more, before a stretch of layers that runs again

A sublayer that can be driven this way offers its ends (``JoinableEnds``).  Every size, constant and tensor name is a
parameter.
"""
import torch

from ..registry import BLOCKS, FEED_FORWARDS, MIXERS, NORMS, STREAM_PARTS
from .base import Block, JoinableEnds, Mixer, Norm, ParamSpec, Part
from .chain_norm_parts import f32_params, linear32, pad_rows


@NORMS.register("offset_rmsnorm")
class OffsetRMSNorm(Norm):
    """out = x / sqrt(mean(x^2) + eps) * (offset + weight), every operation in 32-bit and one rounding at the end; the weight is
    stored around zero.  ``add`` (ops.StreamTerms) and ``again`` (a 32-bit tensor) are added to the stream in the same launch.
    params: size, eps, offset (default 1); name: the weight's checkpoint name (default prefix + "weight")."""

    capturable = True
    accepts_partial_sums = True

    def param_specs(self):
        return [ParamSpec("weight", ((self.params.get("name", self.prefix + "weight"), (self.params["size"],)),), role="bias")]

    def bind(self, tensors):
        w = f32_params(tensors)["weight"]
        super().bind({"weight": (w + float(self.params.get("offset", 1.0))).contiguous()})

    def forward(self, x, out, add=None, rows=None, again=None):
        ops = self.ctx.ops
        ops.stream_terms(x, self.params["eps"], add=ops.StreamTerms.of(add), again=again, weight=self.w["weight"], out=out, rows=rows)
        return out


@STREAM_PARTS.register("embedding_again")
class EmbeddingAgain(Part):
    """What is added to the stream before a pass that runs a stretch of layers again: the embedding's output, kept by the
    model (ModelSpec.keep_embedding)."""

    capturable = True

    def rows(self, step):
        x0 = step.shared.get("embedding_output")
        if x0 is None:
            raise RuntimeError("embedding_again needs the embedding's output: the model's description must set keep_embedding")
        return x0


@BLOCKS.register("parallel_residual")
class ParallelResidual(Block):
    """h = norm(x); x += mixer(h) (+ ffn(h), where the layer has one as a part of its own).  An optional part ``again`` is
    added to x before the norm.  The outputs are handed on un-added (ops.StreamTerms): the stream's next norm adds them."""

    capturable = True
    part_registries = {"again": "stream"}

    def forward(self, step, x, pending):
        p = self.parts
        h = step.ws("normed", (step.rows, x.shape[1]))
        norm = p["norm"]
        norm.forward(x, h, add=pending, again=p["again"].rows(step) if "again" in p else None)
        terms = norm.ctx.ops.StreamTerms.of(p["mixer"].forward(step, h))
        return terms.plus(p["ffn"].forward(step, h)) if "ffn" in p else terms


_REGISTRIES = {"mixer": MIXERS, "ffn": FEED_FORWARDS}


@MIXERS.register("joined_sublayers")
class JoinedSublayers(Mixer):
    """Sublayers that all read the same h, their outputs to be added up.  What they multiply h with is one matrix (their
    sources under one another), what they multiply their last values with is another (side by side): one product in, each
    sublayer's own work between on its columns, one product out whose sum over the columns adds the sublayers up.  A factor
    on a sublayer's output is the sublayer's own (param ``out_factor``): it applies it to the values it hands over, in 32-bit.
    params: members, a tuple of (name, "mixer" | "ffn", PartSpec); the members must offer their ends (JoinableEnds) and are
    built with the param ``joined``."""

    capturable = True

    def __init__(self, params, prefix, ctx):
        super().__init__(params, prefix, ctx)
        self.members, self.sub_part_names = [], []
        for name, registry, spec in params["members"]:
            member = _REGISTRIES[registry].get(spec.kind)({**spec.params, "joined": True}, spec.prefix, ctx)
            if not isinstance(member, JoinableEnds):
                raise ValueError(f"joined_sublayers {prefix!r}: {spec.kind!r} does not offer its ends")
            self.members.append(member)
            self.sub_part_names.append(name)
        if not self.members:
            raise ValueError(f"joined_sublayers {prefix!r}: no members")

    def sub_parts(self):
        return tuple(self.members)

    def param_specs(self):
        sources = tuple(s for m in self.members for s in m.in_sources())
        specs = [ParamSpec("w_in", sources)]
        for name, m in zip(self.sub_part_names, self.members):
            if m.out_source() is not None:
                specs.append(ParamSpec("out_" + name, (m.out_source(),)))
        return specs

    def bind(self, tensors):
        outs = [tensors["out_" + n] for n in self.sub_part_names if "out_" + n in tensors]
        bound = {"w_in": self.ctx.derive(self, "w_in", lambda: pad_rows(tensors["w_in"]))}
        if outs:
            bound["w_out"] = self.ctx.derive(self, "w_out", lambda: torch.cat(outs, 1).contiguous())
        super().bind(bound)

    def forward(self, step, h):
        ops = self.ctx.ops
        proj = linear32(self.ctx, step, h, self.w["w_in"], "joined_in")
        columns = self.w["w_out"].shape[1] if "w_out" in self.w else 0
        values = step.ws("joined_values", (step.rows, columns)) if columns else None
        terms, bias, at, col = [], None, 0, 0
        for m in self.members:
            rows = sum(shape[0] for _, shape in m.in_sources())
            width = m.out_source()[1][1] if m.out_source() is not None else 0
            extra = m.between(step, h, proj[:, at:at + rows], values[:, col:col + width] if width else None)
            if extra is not None:
                terms.append((extra, 1.0))
            if m.out_bias() is not None:
                if bias is not None:
                    raise ValueError(f"joined_sublayers {self.prefix!r}: more than one member has a bias on its output")
                bias = m.out_bias()
            at, col = at + rows, col + width
        if columns:
            terms.insert(0, (linear32(self.ctx, step, values, self.w["w_out"], "joined_out", keep_partial=True), 1.0))
        return ops.StreamTerms(terms, bias)
