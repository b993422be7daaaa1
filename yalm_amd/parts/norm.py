"""RMSNorm: out = x * rsqrt(mean(x^2) + eps) * weight, sums in float32
(src/infer.cpp:136-146, src/infer.cu:525-539).  The parameter `tensor` names the weight behind the
part's prefix (default "weight"); with `offset` c the stored tensor is the weight's distance from c (weight = c +
stored, formed in float32 and kept so, whatever the compute dtype: the sum has no bfloat16 of its own).  `join` is
the norm of a layer that norms a sublayer's OUTPUT: x += norm(y).

LayerNorm: out = (x - mean) / sqrt(mean of the squared deviations + eps) * weight + bias, everything in float32; the bias is
the tensor of the weight's name with `bias_suffix` (default ".b") behind it.  Its `join` norms the SUM of the stream,
times `stream_scale` (default 1), and the sublayer's result: x = norm(stream_scale x + y).

DynamicTanh stands in a norm's place and forms no mean: out = tanh(alpha x) * weight + bias, everything in float32; alpha is one
number, the tensor of the weight's name with `alpha_suffix` (default ".alpha") behind it, the bias as LayerNorm's.  Its `join`
adds the squashed result of a sublayer, times `result_scale` (default 1): x += result_scale norm(y)."""
import torch

from ..ops import kernels
from ..weights.loader import ParamSpec, place
from .base import Part, part


@part("norm", "rmsnorm")
class RMSNorm(Part):
    def __init__(self, spec, dim, prefix):
        super().__init__(spec, dim, prefix)
        self.eps = float(spec.params["eps"])
        self.tensor = self.prefix + str(spec.params.get("tensor", "weight"))
        self.offset = float(spec.params.get("offset", 0.0) or 0.0)
        self.weight = None

    def param_specs(self):
        return [ParamSpec(self.tensor, (self.dim,), init="norm_offset" if self.offset else "norm")]

    def load(self, get, compute_dtype, device):
        if self.offset:
            self.weight = (get(self.tensor).to(torch.float32) + self.offset).to(device).contiguous()
        else:
            self.weight = place(get(self.tensor), compute_dtype, device)
        self.weight_f32 = self.weight if self.weight.dtype == torch.float32 else self.weight.float()

    def weight_bytes(self):
        return self.weight.numel() * self.weight.element_size()

    def fused(self):
        """(float32 weight, eps) for a consumer that folds this norm into its first product."""
        return self.weight_f32, self.eps

    def forward(self, x, out, ctx, row_index=None):
        return kernels.rmsnorm(x, self.weight, out, self.eps, row_index)

    def can_hand_to(self, next_norm):
        """True if `join` can apply next_norm to the stream it leaves."""
        return hasattr(next_norm, "fused")

    def join(self, y, x, ctx, h_out=None, next_norm=None):
        """x += norm(y) (both float32 [T, dim]); h_out, if given, receives the new x in the compute dtype, or with
        next_norm (a norm that offers fused()) that norm's output for the new x."""
        return kernels.norm_add(y, self.weight, self.eps, x, h_out, None if next_norm is None else next_norm.fused())


@part("norm", "layernorm")
class LayerNorm(Part):
    def __init__(self, spec, dim, prefix):
        super().__init__(spec, dim, prefix)
        self.eps = float(spec.params["eps"])
        self.tensor = self.prefix + str(spec.params.get("tensor", "weight"))
        self.bias_tensor = self.tensor + str(spec.params.get("bias_suffix", ".b"))
        self.stream_scale = float(spec.params.get("stream_scale", 1.0))
        self.weight = self.bias = None

    def param_specs(self):
        return [ParamSpec(self.tensor, (self.dim,), init="norm"), ParamSpec(self.bias_tensor, (self.dim,), init="bias")]

    def load(self, get, compute_dtype, device):
        self.weight, self.bias = (get(n).to(torch.float32).to(device).contiguous() for n in (self.tensor, self.bias_tensor))

    def weight_bytes(self):
        return 2 * self.dim * 4

    def joined(self):
        """(weight, bias, eps) for a norm whose `join` applies this one to the stream it leaves."""
        return self.weight, self.bias, self.eps

    def forward(self, x, out, ctx, row_index=None):
        return kernels.layer_norm(x, self.weight, self.bias, self.eps, out, row_index)

    def join(self, y, x, ctx, h_out=None, next_norm=None):
        """x = norm(stream_scale x + y) (both float32 [T, dim]); h_out, if given, receives the new x in the compute dtype,
        or with next_norm (a LayerNorm) that norm's output for the new x."""
        return kernels.layer_norm_sum(y, self.weight, self.bias, self.eps, self.stream_scale, x, h_out,
                                      None if next_norm is None else next_norm.joined())

    def can_hand_to(self, next_norm):
        """True if `join` can apply next_norm to the stream it leaves."""
        return hasattr(next_norm, "joined")


@part("norm", "dynamic_tanh")
class DynamicTanh(Part):
    def __init__(self, spec, dim, prefix):
        super().__init__(spec, dim, prefix)
        self.tensor = self.prefix + str(spec.params.get("tensor", "weight"))
        self.bias_tensor = self.tensor + str(spec.params.get("bias_suffix", ".b"))
        self.alpha_tensor = self.tensor + str(spec.params.get("alpha_suffix", ".alpha"))
        self.result_scale = float(spec.params.get("result_scale", 1.0))
        self.weight = self.bias = self.alpha = None

    def param_specs(self):
        return [ParamSpec(self.tensor, (self.dim,), init="norm"), ParamSpec(self.bias_tensor, (self.dim,), init="bias"),
                ParamSpec(self.alpha_tensor, (), init="fraction")]

    def load(self, get, compute_dtype, device):
        self.weight, self.bias = (get(n).to(torch.float32).to(device).contiguous() for n in (self.tensor, self.bias_tensor))
        self.alpha = float(get(self.alpha_tensor))

    def weight_bytes(self):
        return 2 * self.dim * 4

    def squash(self):
        """(alpha, weight, bias) for a norm whose `join` applies this one to the stream it leaves."""
        return self.alpha, self.weight, self.bias

    def forward(self, x, out, ctx, row_index=None):
        return kernels.squash(x, *self.squash(), out, row_index)

    def join(self, y, x, ctx, h_out=None, next_norm=None, y_bias=None):
        """x += result_scale norm(y + y_bias) (x, y float32 [T, dim]; y_bias float32 [dim] or None); h_out, if given, receives the
        new x in the compute dtype, or with next_norm (a DynamicTanh) that norm's output for the new x."""
        return kernels.squash_add(y, *self.squash(), self.result_scale, x, h_out, None if next_norm is None else next_norm.squash(), y_bias)

    def can_hand_to(self, next_norm):
        """True if `join` can apply next_norm to the stream it leaves."""
        return hasattr(next_norm, "squash")
