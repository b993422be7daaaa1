"""Lightning attention as a mixer: a linear attention whose state decays by one fixed number a head.  Per head a state S
[key_dim, value_dim] in float32, zero for a new sequence and kept from one step to the next in the cache's fixed-size
per-sequence state.

Per token: q = silu(W_q h) and k = silu(W_k h) (`n_heads` heads of `key_dim`), v = silu(W_v h) (`n_heads` heads of
`value_dim`); per head, `decay` naming its number g in [0, 1],
    S <- g S + k v^T;   o = S^T q
(no other scale; the read-out sees the token's own write).  The heads' results side by side are divided by their common
root mean square, multiplied by a weight and by sigmoid(W_g h), and W_o carries them to the stream.  q | k | v | g are one product
with float32 results; everything behind it is float32 (ops.kernels.lightning: token by token; lightning_tiles, steps of
prompts: 64 tokens at a time on the matrix cores)."""
import torch

from ..cache.manager import StateRequest
from ..ops import kernels
from ..weights.loader import ParamSpec
from .attention import kv_tiles
from .base import JoinableMixer, part

NAMES = {"q": "q", "k": "k", "v": "v", "gate": "g", "norm": "norm", "out": "o"}
TILES_MIN_TOKENS = 32            # tokens a sequence (on average) from which a step of prompts goes tile by tile


@part("mixer", "lightning")
class LightningAttention(JoinableMixer):
    prompt_tables = (kv_tiles,)
    joinable = True

    def __init__(self, spec, dim, prefix):
        super().__init__(spec, dim, prefix)
        p = spec.params
        self.n_heads = int(p["n_heads"])
        self.key_dim = int(p["key_dim"])
        self.value_dim = int(p.get("value_dim") or self.key_dim)
        self.decay = [float(g) for g in p["decay"]]
        self.eps = float(p.get("eps", 1e-6))
        if self.n_heads <= 0 or not 0 < self.key_dim <= kernels.LIGHTNING_MAX_KEY_DIM or self.value_dim <= 0 \
                or len(self.decay) != self.n_heads or not all(0.0 <= g <= 1.0 for g in self.decay):
            raise ValueError("lightning attention: %d heads with keys of %d (at most %d), values of %d and the decays %r are not offered"
                             % (self.n_heads, self.key_dim, kernels.LIGHTNING_MAX_KEY_DIM, self.value_dim, self.decay))
        self.names = dict(NAMES)
        self.names.update(p.get("tensors") or {})
        self.qk = self.n_heads * self.key_dim
        self.vv = self.n_heads * self.value_dim
        self.powers = self.w_norm = None

    def _n(self, key):
        return self.prefix + self.names[key]

    def param_specs(self):
        D = self.dim
        return [ParamSpec(self._n("q"), (self.qk, D), fan_in=D), ParamSpec(self._n("k"), (self.qk, D), fan_in=D),
                ParamSpec(self._n("v"), (self.vv, D), fan_in=D), ParamSpec(self._n("gate"), (self.vv, D), fan_in=D),
                ParamSpec(self._n("norm"), (self.vv,), init="norm"), ParamSpec(self._n("out"), (D, self.vv), fan_in=self.vv)]

    @property
    def n_in(self):
        return 2 * self.qk + 2 * self.vv

    @property
    def n_out(self):
        return self.vv

    def in_rows(self, get):
        return torch.cat([get(self._n(k)) for k in ("q", "k", "v", "gate")], dim=0)

    def out_columns(self, get):
        return get(self._n("out"))

    def load_rest(self, get, compute_dtype, device, scale=1.0):
        self.w_norm = (get(self._n("norm")).to(torch.float32).reshape(-1) * scale).to(device).contiguous()
        g = torch.tensor(self.decay, dtype=torch.float64)
        self.powers = (g[:, None] ** torch.arange(kernels.LIGHTNING_POWERS, dtype=torch.float64)).to(torch.float32).to(device).contiguous()

    def cache_request(self):
        return StateRequest((kernels.lightning_state_elements(self.n_heads, self.key_dim, self.value_dim),), torch.float32)

    def row_elements(self):
        padded = next((p for p in (32, 64, 128) if p >= self.key_dim), 0)          # a scaled query's row in lightning_tiles
        return max(self.n_in, self.n_heads * padded)

    def describe(self, compute_dtype):
        return "lightning attention, %d heads of %d x %d: float32, prompts by tiles of 64 tokens on the matrix cores, single tokens " \
               "with state columns in the registers of a group of lanes" % (self.n_heads, self.key_dim, self.value_dim), False

    def between(self, h, proj, o, ctx, line, writes_cache, scale=1.0):
        T, ws = proj.shape[0], ctx.ws
        sizes = (self.n_heads, self.key_dim, self.value_dim)
        z, gate = proj[:, :2 * self.qk + self.vv], proj[:, 2 * self.qk + self.vv:]
        raw = ws.get("lightning.raw", (T, self.vv), torch.float32)
        state = ctx.cache.group_of(line).line_state(line)
        if ctx.mode == "prefill" and T >= TILES_MIN_TOKENS * ctx.seq_slot.shape[0] and not kernels.FORCE_SIMPLE \
                and kernels.lightning_tiles_fit(self.key_dim):
            tiles = ctx.tables["kv_tiles"]
            kernels.lightning_tiles(z, self.powers, state, raw, ctx.cu_seqlens, ctx.seq_slot, tiles["seq_tile0"], tiles["n_tiles"],
                                    *sizes, ws.get)
        else:
            kernels.lightning(z, self.powers, state, raw, ctx.cu_seqlens, ctx.seq_slot, *sizes)
        kernels.rms_gate(raw, self.w_norm, self.eps, gate, o)         # the mixer's share rides on the norm's weights
