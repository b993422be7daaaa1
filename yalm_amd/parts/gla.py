"""Gated linear attention as a mixer: per head a state S [key_dim, value_dim] in float32, zero for a new sequence and kept
from one step to the next in the cache's fixed-size per-sequence state.

Per token: q = W_q h q_scale and k = W_k h (`n_heads` heads of `key_dim`), v = W_v h (`n_heads` heads of `value_dim`), and
a decay per head and key channel f = sigmoid(W_2 (W_1 h) + b)^(1 / tau), the inner size of that product being `decay_rank`;
per head
    S <- diag(f) S + k v^T;   o = S^T q
(the read-out sees the token's own write).  Each head's o is divided by its root mean square, multiplied by a weight
shared by the heads and by silu(W_g h), and W_o carries the heads to the stream.  q | k | v | g | W_1 h are one product
with float32 results; everything behind it is float32, the small product with W_2 included (ops.kernels.gla: token by
token; gla_tiles, steps of prompts: 64 tokens at a time on the matrix cores)."""
import torch

from ..cache.manager import StateRequest
from ..ops import kernels
from ..weights.loader import ParamSpec, place
from .attention import kv_tiles
from .base import Part, part

NAMES = {"q": "q", "k": "k", "v": "v", "gate": "g", "decay_in": "a1", "decay_out": "a2", "decay_bias": "a2.b", "norm": "norm",
         "out": "o"}


@part("mixer", "gla")
class GatedLinearAttention(Part):
    prompt_tables = (kv_tiles,)

    def __init__(self, spec, dim, prefix):
        super().__init__(spec, dim, prefix)
        p = spec.params
        self.n_heads = int(p["n_heads"])
        self.key_dim = int(p["key_dim"])
        self.value_dim = int(p.get("value_dim") or self.key_dim)
        self.decay_rank = int(p["decay_rank"])
        self.tau = float(p.get("tau", 16.0))
        self.q_scale = float(p.get("q_scale") or self.key_dim ** -0.5)
        self.eps = float(p.get("eps", 1e-6))
        if self.n_heads <= 0 or not 0 < self.key_dim <= kernels.GLA_MAX_KEY_DIM or self.value_dim <= 0 \
                or not 0 < self.decay_rank <= kernels.GLA_MAX_RANK or not self.tau > 0:
            raise ValueError("gated linear attention: %d heads with keys of %d (at most %d), values of %d, decays of rank %d (at "
                             "most %d) and tau %g are not offered" % (self.n_heads, self.key_dim, kernels.GLA_MAX_KEY_DIM,
                                                                      self.value_dim, self.decay_rank, kernels.GLA_MAX_RANK, self.tau))
        self.names = dict(NAMES)
        self.names.update(p.get("tensors") or {})
        self.qk = self.n_heads * self.key_dim
        self.vv = self.n_heads * self.value_dim
        self.proj_cols = 2 * self.qk + 2 * self.vv + self.decay_rank
        self.w_in = self.wo = self.w2 = self.decay_bias = self.w_norm = None

    def _n(self, key):
        return self.prefix + self.names[key]

    def param_specs(self):
        D, r = self.dim, self.decay_rank
        return [ParamSpec(self._n("q"), (self.qk, D), fan_in=D), ParamSpec(self._n("k"), (self.qk, D), fan_in=D),
                ParamSpec(self._n("v"), (self.vv, D), fan_in=D), ParamSpec(self._n("gate"), (self.vv, D), fan_in=D),
                ParamSpec(self._n("decay_in"), (r, D), fan_in=D), ParamSpec(self._n("decay_out"), (self.qk, r), fan_in=r),
                ParamSpec(self._n("decay_bias"), (self.qk,), init="bias"),
                ParamSpec(self._n("norm"), (self.value_dim,), init="norm"), ParamSpec(self._n("out"), (D, self.vv), fan_in=self.vv)]

    def load(self, get, compute_dtype, device):
        def f32(key):
            return get(self._n(key)).to(torch.float32)
        self.w_in = place(torch.cat([get(self._n(k)) for k in ("q", "k", "v", "gate", "decay_in")], dim=0), compute_dtype, device)
        self.wo = place(get(self._n("out")), compute_dtype, device)
        # the recurrence's kernel takes W_2 in float32, rounded to the compute dtype as every other matrix is
        w2 = torch.zeros((self.qk, kernels.gla_padded_rank(self.decay_rank)), dtype=torch.float32)
        w2[:, :self.decay_rank] = get(self._n("decay_out")).to(compute_dtype).to(torch.float32)
        self.w2 = w2.to(device).contiguous()
        self.decay_bias = f32("decay_bias").reshape(-1).to(device).contiguous()
        self.w_norm = f32("norm").reshape(-1).to(device).contiguous()

    def weight_bytes(self):
        return (self.w_in.numel() + self.wo.numel()) * self.w_in.element_size() + self.w2.numel() * 4

    def cache_request(self):
        return StateRequest((kernels.gla_state_elements(self.n_heads, self.key_dim, self.value_dim),), torch.float32)

    def row_elements(self):
        padded = next((p for p in (32, 64, 128) if p >= self.key_dim), 0)          # a scaled query's row in gla_tiles
        return max(self.proj_cols, self.n_heads * padded)

    def describe(self, compute_dtype):
        return "gated linear attention, %d heads of %d x %d, decays of rank %d: float32, prompts by tiles of 64 tokens on the " \
               "matrix cores, single tokens with state columns in the registers of a group of lanes" % (self.n_heads, self.key_dim, self.value_dim, self.decay_rank), False

    def forward(self, h, x, ctx, line, writes_cache=True):
        """Adds the mixer's result to the stream x."""
        return self._run(h, x, ctx, line, kernels.EPI_ADD_F32)

    def forward_to(self, h, y, ctx, line, writes_cache=True):
        """Writes the mixer's result to y (float32 [T, dim])."""
        return self._run(h, y, ctx, line, kernels.EPI_STORE_F32)

    def _run(self, h, x, ctx, line, epilogue):
        T = h.shape[0]
        ws = ctx.ws
        proj = ws.get("gla.proj", (T, self.proj_cols), torch.float32)
        self._gemm(ctx, h, self.w_in, proj, kernels.EPI_STORE_F32)
        raw = ws.get("gla.raw", (T, self.vv), torch.float32)
        o = ws.get("gla.o", (T, self.vv), h.dtype)
        state = ctx.cache.group_of(line).line_state(line)
        B = ctx.seq_slot.shape[0]
        sizes = (self.n_heads, self.key_dim, self.value_dim, self.decay_rank, self.q_scale, self.tau, self.eps)
        # With float32 as the compute dtype prompts go token by token too: the decays' products are then formed one factor
        # at a time, without the rounding of their logarithms' sums.
        if ctx.mode == "prefill" and h.dtype == torch.bfloat16 and T >= kernels.GLA_TILES_MIN_TOKENS * B and not kernels.FORCE_SIMPLE \
                and kernels.gla_tiles_fit(self.key_dim, self.decay_rank):
            tiles = ctx.tables["kv_tiles"]
            kernels.gla_tiles(proj, self.w2, self.decay_bias, self.w_norm, state, raw, ctx.cu_seqlens, ctx.seq_slot,
                              tiles["seq_tile0"], tiles["n_tiles"], o, *sizes, ws.get)
        else:
            kernels.gla(proj, self.w2, self.decay_bias, self.w_norm, state, raw, ctx.cu_seqlens, ctx.seq_slot, o, *sizes)
        self._gemm(ctx, o, self.wo, x, epilogue)
