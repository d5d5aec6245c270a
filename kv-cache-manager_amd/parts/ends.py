"""How a sublayer that offers its ends (base.JoinableEnds) runs on its own: its first product, its own work, its last one."""
from .base import JoinableEnds, Mixer, ParamSpec
from .chain_norm_parts import f32_params, linear32, pad_rows


class EndsMixer(JoinableEnds, Mixer):
    """A mixer that offers its ends.  With the param ``joined`` its first and last product are whoever drives it's own."""

    ends_name = "ends"      # names the work buffers of the mixer run on its own

    @property
    def joined(self):
        return bool(self.params.get("joined"))

    def own_specs(self):
        """Tensors beside the two matrices."""
        return []

    def param_specs(self):
        ends = [] if self.joined else [ParamSpec("w_in", self.in_sources()), ParamSpec("w_out", (self.out_source(),))]
        return ends + self.own_specs()

    def bind(self, tensors):
        ends = {k: tensors[k] for k in ("w_in", "w_out") if k in tensors}
        if "w_in" in ends:
            ends["w_in"] = self.ctx.derive(self, "w_in", lambda: pad_rows(tensors["w_in"]))
        super().bind({**f32_params({k: v for k, v in tensors.items() if k not in ends}), **ends})

    def forward(self, step, h):
        proj = linear32(self.ctx, step, h, self.w["w_in"], self.ends_name + "_in")
        values = step.ws(self.ends_name + "_values", (step.rows, self.w["w_out"].shape[1]))
        self.between(step, h, proj, values)
        return linear32(self.ctx, step, values, self.w["w_out"], self.ends_name + "_out", keep_partial=True)      # the stream's next norm adds the slices
