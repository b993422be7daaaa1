"""Two mixers side by side as one mixer: both read the same input, each result is normed over the model's width
(RMS, a plain weight of its own), and `weight` times their sum goes to the stream (`weight` 1/2: their mean).  With `scales`
(left, right) the results are not normed: the mixer's result is left * (the left one's) + right * (the right one's).  The two
(JoinableMixer, both joinable) then share one product in front and one behind: their first matrices stand one below the other,
their last ones side by side, and a side's scale rides on what it puts in front of the last product (in float32, before that is
rounded to the compute dtype).

The two are any registered mixers that offer forward_to (which writes a result instead of adding it); each keeps what
it keeps (keys and values in pages, a fixed-size state) under a cache line of its own: this mixer's cache request is
the pair {"left": ..., "right": ...}, and the cache manager gives line (l, "left") and (l, "right") to the members
of line l."""
import torch

from ..ops import kernels
from ..weights.loader import ParamSpec, place
from .base import JoinableMixer, Part, build_part, part


@part("mixer", "side_by_side")
class SideBySide(Part):
    def __init__(self, spec, dim, prefix):
        super().__init__(spec, dim, prefix)
        p = spec.params
        self.left = build_part("mixer", p["left"], dim, prefix)
        self.right = build_part("mixer", p["right"], dim, prefix)
        for m in (self.left, self.right):
            if not hasattr(m, "forward_to"):
                raise ValueError("a %s cannot stand beside another mixer: it has no forward_to" % type(m).__name__)
        self.eps = float(p.get("eps", 1e-6))
        self.weight = float(p.get("weight", 0.5))
        names = p.get("tensors") or {}
        self.left_norm = self.prefix + str(names.get("left_norm", "left.out"))
        self.right_norm = self.prefix + str(names.get("right_norm", "right.out"))
        self.w_left = self.w_right = None
        self.scales = tuple(float(s) for s in p["scales"]) if p.get("scales") else None
        self.w_in = self.wo = None
        if self.scales is not None:
            for m, scale in zip((self.left, self.right), self.scales):
                if not isinstance(m, JoinableMixer) or not m.joinable:
                    raise ValueError("a %s cannot share its products with another mixer" % type(m).__name__)
                m.joined, m.share = True, scale

    @property
    def late_bias(self):
        """The bias that the joined result lacks: the members' (they have loaded them times their scales)."""
        biases = [m.late_bias for m in (self.left, self.right) if self.scales is not None and m.late_bias is not None]
        return None if not biases else (biases[0] if len(biases) == 1 else biases[0] + biases[1])

    def children(self):
        return [self.left, self.right]

    @property
    def prompt_tables(self):
        return tuple(getattr(self.left, "prompt_tables", ())) + tuple(getattr(self.right, "prompt_tables", ()))

    def param_specs(self):
        if self.scales is not None:
            return []
        return [ParamSpec(self.left_norm, (self.dim,), init="norm"), ParamSpec(self.right_norm, (self.dim,), init="norm")]

    def load(self, get, compute_dtype, device):
        if self.scales is not None:
            self.w_in = place(torch.cat([m.in_rows(get) for m in (self.left, self.right)], dim=0), compute_dtype, device)
            self.wo = place(torch.cat([m.out_columns(get) for m in (self.left, self.right)], dim=1), compute_dtype, device)
            return                        # the members load the rest themselves
        # the share of each side rides on its norm's weight (exact for a power of two)
        self.w_left = (get(self.left_norm).to(torch.float32) * self.weight).to(device).contiguous()
        self.w_right = (get(self.right_norm).to(torch.float32) * self.weight).to(device).contiguous()

    def weight_bytes(self):
        if self.scales is not None:
            return (self.w_in.numel() + self.wo.numel()) * self.w_in.element_size()
        return 2 * self.dim * 4

    def cache_request(self):
        return {"left": self.left.cache_request(), "right": self.right.cache_request()}

    def describe(self, compute_dtype):
        if self.scales is not None:
            return "two mixers side by side, one product in front of both and one behind", False
        return "two mixers side by side, each normed over the width", False

    def row_elements(self):
        return max(self.left.n_in + self.right.n_in, self.left.n_out + self.right.n_out) if self.scales is not None else self.dim

    def forward_to(self, h, y, ctx, line, writes_cache=True, late_bias_taken=False):
        """Writes the mixer's result to y (float32 [T, dim]), without its late_bias."""
        if self.scales is None:
            raise ValueError("two mixers that are normed add to the stream only")
        if self.late_bias is not None and not late_bias_taken:
            raise ValueError("this mixer's result lacks a bias that nobody adds")
        self._joint(h, y, ctx, line, writes_cache, kernels.EPI_STORE_F32)

    def _joint(self, h, x, ctx, line, writes_cache, epilogue):
        T, l, r = h.shape[0], self.left, self.right
        proj = ctx.ws.get("side.proj", (T, l.n_in + r.n_in), torch.float32)
        self._gemm(ctx, h, self.w_in, proj, kernels.EPI_STORE_F32)
        o = ctx.ws.get("side.o", (T, l.n_out + r.n_out), h.dtype)
        l.between(h, proj[:, :l.n_in], o[:, :l.n_out], ctx, (line, "left"), writes_cache, l.share)
        r.between(h, proj[:, l.n_in:], o[:, l.n_out:], ctx, (line, "right"), writes_cache, r.share)
        self._gemm(ctx, o, self.wo, x, epilogue)

    def forward(self, h, x, ctx, line, writes_cache=True):
        T = h.shape[0]
        if self.scales is not None:
            if self.late_bias is not None:
                raise ValueError("a mixer whose last product has a bias writes its result (forward_to); it does not add to the stream")
            return self._joint(h, x, ctx, line, writes_cache, kernels.EPI_ADD_F32)
        y = ctx.ws.get("side.y", (T, self.dim), torch.float32)
        self.left.forward_to(h, y, ctx, (line, "left"), writes_cache)
        kernels.norm_add(y, self.w_left, self.eps, x)
        self.right.forward_to(h, y, ctx, (line, "right"), writes_cache)
        kernels.norm_add(y, self.w_right, self.eps, x)
