"""Griffin's recurrent block as a mixer: a gated linear recurrence on every channel, behind a short convolution and beside a
gelu branch.  Per token, with `width` channels in `blocks` equal blocks:
    y = gelu(W_y h + y0),   u = conv(W_x h + x0) + c0         (causal, `taps` taps a channel, the last one the token's own)
    r = sigmoid(R_b u_b + r0),   i = sigmoid(I_b u_b + i0)    (one pair of matrices a block)
    a = exp(-rate r softplus(lam));   S <- a S + sqrt(1 - a^2) i u
and W_o carries S y to the stream (gelu in its tanh form; `rate` defaults to 8).  S and the convolution's last taps - 1 inputs are float32, zero for a
new sequence, and kept in the cache's fixed-size per-sequence state under two lines of the layer's.  W_y | W_x are one product
with float32 results; everything behind it is float32 (ops.kernels.time_conv, lru, lru_step)."""
import torch

from ..cache.manager import StateRequest
from ..ops import kernels
from ..weights.loader import ParamSpec, place
from .attention import kv_tiles
from .base import Part, part

NAMES = {"y": "y", "x": "x", "y_bias": "y.b", "x_bias": "x.b", "conv": "conv", "conv_bias": "conv.b", "r": "ra", "r_bias": "ra.b",
         "i": "ri", "i_bias": "ri.b", "lam": "lam", "out": "o"}


@part("mixer", "rglru")
class GatedLinearRecurrentUnit(Part):
    prompt_tables = (kv_tiles,)

    def __init__(self, spec, dim, prefix):
        super().__init__(spec, dim, prefix)
        p = spec.params
        self.width = int(p.get("width") or dim)
        self.blocks = int(p["blocks"])
        self.taps = int(p["taps"])
        self.rate = float(p.get("rate", 8.0))
        if self.width <= 0 or self.blocks <= 0 or self.width % self.blocks or not 0 < self.taps <= kernels.TIME_CONV_MAX_TAPS:
            raise ValueError("gated linear recurrence: %d channels in %d blocks behind %d taps (at most %d) are not offered"
                             % (self.width, self.blocks, self.taps, kernels.TIME_CONV_MAX_TAPS))
        self.names = dict(NAMES)
        self.names.update(p.get("tensors") or {})
        self.w_in = self.wo = self.w_gates = None
        self.y_bias = self.x_bias = self.conv_w = self.conv_bias = self.gate_bias = self.slope = None

    def _n(self, key):
        return self.prefix + self.names[key]

    def param_specs(self):
        D, W, nb = self.dim, self.width, self.blocks
        n = W // nb
        out = [ParamSpec(self._n(k), (W, D), fan_in=D) for k in ("y", "x")]
        out += [ParamSpec(self._n(k), (W,), init="bias") for k in ("y_bias", "x_bias", "conv_bias")]
        out.append(ParamSpec(self._n("conv"), (W, self.taps), init="taps"))
        out += [ParamSpec(self._n(k), (nb, n, n), fan_in=n) for k in ("r", "i")]
        out += [ParamSpec(self._n(k), (nb, n), init="bias") for k in ("r_bias", "i_bias")]
        return out + [ParamSpec(self._n("lam"), (W,), init="decay_log"), ParamSpec(self._n("out"), (D, W), fan_in=W)]

    def load(self, get, compute_dtype, device):
        def f32(key):
            return get(self._n(key)).to(torch.float32).reshape(-1).to(device).contiguous()
        self.w_in = place(torch.cat([get(self._n("y")), get(self._n("x"))], dim=0), compute_dtype, device)
        self.wo = place(get(self._n("out")), compute_dtype, device)
        self.w_gates = place(torch.stack([get(self._n("r")), get(self._n("i"))]), compute_dtype, device)
        self.y_bias, self.x_bias, self.conv_bias = f32("y_bias"), f32("x_bias"), f32("conv_bias")
        self.gate_bias = torch.stack([f32("r_bias"), f32("i_bias")]).contiguous()
        self.conv_w = get(self._n("conv")).to(torch.float32).t().contiguous().to(device)             # tap by tap: [taps, width]
        lam = get(self._n("lam")).to(torch.float64).reshape(-1)
        self.slope = (-self.rate * torch.nn.functional.softplus(lam, threshold=1e9)).to(torch.float32).to(device).contiguous()

    def weight_bytes(self):
        return (self.w_in.numel() + self.wo.numel() + self.w_gates.numel()) * self.w_in.element_size()

    def cache_request(self):
        return {"conv": StateRequest((self.taps - 1, self.width), torch.float32) if self.taps > 1 else None,
                "state": StateRequest((self.width,), torch.float32)}

    def row_elements(self):
        return 2 * self.width

    def describe(self, compute_dtype):
        return "gated linear recurrence on %d channels in %d blocks, %d taps in front: float32" % (self.width, self.blocks, self.taps), False

    def forward(self, h, x, ctx, line, writes_cache=True):
        """Adds the mixer's result to the stream x."""
        return self._run(h, x, ctx, line, kernels.EPI_ADD_F32)

    def forward_to(self, h, y, ctx, line, writes_cache=True):
        """Writes the mixer's result to y (float32 [T, dim])."""
        return self._run(h, y, ctx, line, kernels.EPI_STORE_F32)

    def _run(self, h, x, ctx, line, epilogue):
        T, W, ws = h.shape[0], self.width, ctx.ws
        proj = ws.get("rglru.proj", (T, 2 * W), torch.float32)
        self._gemm(ctx, h, self.w_in, proj, kernels.EPI_STORE_F32)
        z, fresh = proj[:, :W], proj[:, W:]
        carried = ctx.cache.group_of((line, "conv")).line_state((line, "conv")) if self.taps > 1 else None
        u = ws.get("rglru.u", (T, W), torch.float32)
        kernels.time_conv(fresh, self.conv_w, carried, u, ctx.tok_seq, ctx.cu_seqlens, ctx.seq_slot, residual=False,
                          one_token_each=ctx.mode == "decode", in_bias=self.x_bias, bias=self.conv_bias)
        state = ctx.cache.group_of((line, "state")).line_state((line, "state"))
        o = ws.get("rglru.o", (T, W), h.dtype)
        gates = (self.w_gates, self.gate_bias, self.slope, z, self.y_bias, state, o)
        if ctx.mode == "prefill":
            tiles = ctx.tables["kv_tiles"]
            kernels.lru(u, *gates, ctx.tok_seq, ctx.cu_seqlens, ctx.seq_slot, ws.get, tiles["seq_tile0"], tiles["n_tiles"])
        elif T > kernels.LRU_STEP_MAX_ROWS and h.dtype == torch.bfloat16:
            kernels.lru(u, *gates, ctx.tok_seq, ctx.cu_seqlens, ctx.seq_slot, ws.get)
        else:
            kernels.lru_step(u, *gates, ctx.seq_slot)
        self._gemm(ctx, o, self.wo, x, epilogue)
