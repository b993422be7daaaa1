"""Mixture of experts: `n_experts` small feed-forwards, of which a token uses the `top` whose router
scores are largest.

Router: s = softmax(W_router h (+ a bias, the tensor `router_bias`)) over all experts, in float32; the chosen experts'
weights are their scores (`renormalize`: divided by their sum; "chosen": the experts with the largest logits, weighted
by the softmax over the chosen logits alone).  Expert: g = min(W_gate h, limit), u = clamp(W_up h, -limit, limit),
out = W_down (g sigmoid(alpha g) (u + up_shift)) (limit 0: no clamping; up_shift defaults to 1; alpha 1 and up_shift 0
make silu(gate) * up).  The part's result is the weighted sum over
a token's chosen experts, in the order of their scores.  `unit` "relu2": experts of two matrices, out = W_down
relu(W_up h)^2.  `scores` "sigmoid": s = sigmoid(W_router h); experts are chosen by s plus a correction (the tensor
`correction`, one number an expert), among the `keep_groups` best of `groups` equal groups of neighbouring experts (a
group's score is the sum of its two largest corrected scores, or with `group_score` "max" its largest), and weigh s over the sum
of the chosen s, times `weight_scale`.  Softmax scores with `renormalize` take a correction, groups and weight_scale likewise.  With `shared` = {hidden, prefix, gate} one more expert of the
same form (its tensors behind `prefix`, its own hidden size) runs for every token and is added, times sigmoid(w . h), one
number a token (w: the tensor `gate` behind the prefix, [1, width]; no `gate`: added as it is).

The experts' matrices are stacked at load ([E, F, D], [E, F, D], [E, D, F]); routing happens on the device
(nothing of it reaches the host, so a decode step stays a captured graph), and every (token, choice) pair is
served from its expert's weights.  A step of GROUPED_MIN_ROWS rows or more (bfloat16; whole prompts, and decode
batches of 16 and more) groups the pairs by expert instead and multiplies every expert's rows as tiles on the
matrix cores, all experts in one launch a product: the grouped products read every chosen expert once while the
pairs would read it once a pair (measured at width 4,096, 32 experts of 2,048,
4 a token, four layers: batch 8 1.01 against 1.03 ms a step, batch 16 1.46 against 1.15, batch 64 3.32 against 1.44,
batch 128 5.54 against 1.60).  Both ways are decided on the device, so a decode step stays a captured graph."""
import torch

from ..ops import kernels
from ..weights.loader import ParamSpec, place
from .base import Part, part
from .swiglu import interleave_gate_up


GROUPED_MIN_ROWS = 9             # steps of this many rows and more group the pairs by expert


@part("feed_forward", "moe")
class MixtureOfExperts(Part):
    def __init__(self, spec, dim, prefix):
        super().__init__(spec, dim, prefix)
        p = spec.params
        self.hidden = int(p["hidden"])
        self.n_experts = int(p["n_experts"])
        self.top = int(p["top"])
        self.limit = float(p.get("limit", 0.0) or 0.0)
        self.alpha = float(p.get("alpha", 1.0))
        self.up_shift = float(p.get("up_shift", 1.0))
        self.renormalize = p.get("renormalize", False)
        self.renormalize = "chosen" if self.renormalize == "chosen" else bool(self.renormalize)
        self.expert_prefix = str(p.get("expert_prefix", "experts.%d."))
        self.gated = p.get("unit", "gated") == "gated"
        self.sigmoid = p.get("scores", "softmax") == "sigmoid"
        if p.get("unit", "gated") not in ("gated", "relu2") or p.get("scores", "softmax") not in ("softmax", "sigmoid"):
            raise ValueError("mixture of experts: unit %r with scores %r is not offered" % (p.get("unit"), p.get("scores")))
        self.groups, self.keep_groups = int(p.get("groups", 1)), int(p.get("keep_groups", 1))
        self.weight_scale = float(p.get("weight_scale", 1.0))
        self.names = {"router": "router", "gate": "gate", "up": "up", "down": "down"}
        self.names.update(p.get("tensors") or {})
        self.router_bias = self.names.get("router_bias")           # a tensor's name, or no bias
        if not 0 < self.top <= self.n_experts or self.n_experts > kernels.MOE_MAX_EXPERTS:
            raise ValueError("mixture of experts: %d of %d experts is not offered (at most %d experts)"
                             % (self.top, self.n_experts, kernels.MOE_MAX_EXPERTS))
        if self.groups <= 0 or self.n_experts % self.groups or not 0 < self.keep_groups <= self.groups \
                or self.top > self.keep_groups * (self.n_experts // self.groups):
            raise ValueError("mixture of experts: %d of %d experts from %d of %d groups is not offered"
                             % (self.top, self.n_experts, self.keep_groups, self.groups))
        self.correction_name = self.names.get("correction")        # a tensor's name, or no correction
        if p.get("group_score", "top2") not in ("top2", "max"):
            raise ValueError("mixture of experts: a group's score %r is neither 'top2' nor 'max'" % (p.get("group_score"),))
        self.group_max = p.get("group_score", "top2") == "max"
        # whether the choice is made by corrected scores inside groups (a kernel of its own)
        self.corrected = self.sigmoid or self.groups > 1 or self.weight_scale != 1.0 or bool(self.correction_name)
        if self.corrected and not self.sigmoid and (self.renormalize is not True or self.router_bias):
            raise ValueError("groups, a correction and weight_scale go with sigmoid scores, or with softmax scores brought to one sum")
        if self.sigmoid and (self.renormalize or self.router_bias):
            raise ValueError("sigmoid scores are always brought to one sum and take no router bias")
        self.correction = None
        self.w_router = self.w_gate = self.w_up = self.w_down = self.b_router = None
        self.shared = None
        if p.get("shared"):
            s = p["shared"]
            if self.limit or self.alpha != 1.0 or self.up_shift:
                raise ValueError("a shared expert is silu(gate) * up: it goes with limit 0, alpha 1 and up_shift 0")
            self.shared = {"hidden": int(s["hidden"]), "prefix": str(s.get("prefix", "shared.")), "gate": s.get("gate")}
        self.ws_gate_up = self.ws_down = self.ws_gate = None

    def _expert(self, e, key):
        return self.prefix + (self.expert_prefix % e) + self.names[key]

    def param_specs(self):
        D, F = self.dim, self.hidden
        out = [ParamSpec(self.prefix + self.names["router"], (self.n_experts, D), fan_in=D)]
        if self.router_bias:
            out.append(ParamSpec(self.prefix + self.router_bias, (self.n_experts,), init="bias"))
        if self.correction_name:
            out.append(ParamSpec(self.prefix + self.correction_name, (self.n_experts,), init="bias"))
        for e in range(self.n_experts):
            if self.gated:
                out.append(ParamSpec(self._expert(e, "gate"), (F, D), fan_in=D))
            out += [ParamSpec(self._expert(e, "up"), (F, D), fan_in=D), ParamSpec(self._expert(e, "down"), (D, F), fan_in=F)]
        if self.shared:
            Fs = self.shared["hidden"]
            out += [ParamSpec(self._shared("gate"), (Fs, D), fan_in=D), ParamSpec(self._shared("up"), (Fs, D), fan_in=D),
                    ParamSpec(self._shared("down"), (D, Fs), fan_in=Fs)]
            if self.shared["gate"]:
                out.append(ParamSpec(self.prefix + self.shared["prefix"] + self.shared["gate"], (1, D), fan_in=D))
        return out

    def _shared(self, key):
        return self.prefix + self.shared["prefix"] + self.names[key]

    def load(self, get, compute_dtype, device):
        E = self.n_experts
        self.w_router = place(get(self.prefix + self.names["router"]), compute_dtype, device)
        if self.router_bias:
            self.b_router = get(self.prefix + self.router_bias).to(torch.float32).to(device).contiguous()
        if self.correction_name:
            self.correction = get(self.prefix + self.correction_name).to(torch.float32).to(device).contiguous()
        if self.gated:
            self.w_gate = place(torch.stack([get(self._expert(e, "gate")) for e in range(E)]), compute_dtype, device)
        self.w_up = place(torch.stack([get(self._expert(e, "up")) for e in range(E)]), compute_dtype, device)
        self.w_down = place(torch.stack([get(self._expert(e, "down")) for e in range(E)]), compute_dtype, device)
        if self.shared:
            self.ws_gate_up = place(interleave_gate_up(get(self._shared("gate")), get(self._shared("up"))), compute_dtype, device)
            self.ws_down = place(get(self._shared("down")), compute_dtype, device)
            if self.shared["gate"]:
                w = get(self.prefix + self.shared["prefix"] + self.shared["gate"]).reshape(-1)
                self.ws_gate = w.to(device=device, dtype=compute_dtype).contiguous()     # the activations' dtype

    def weight_bytes(self):
        """What a token's step reads: the router, `top` experts and the shared expert."""
        item = self.w_down.element_size()
        shared = (3 * self.shared["hidden"] + 1) * self.dim if self.shared else 0
        return (self.n_experts * self.dim + self.top * self.matrices() * self.hidden * self.dim + shared) * item

    def matrices(self):
        """Matrices an expert has."""
        return 3 if self.gated else 2

    def row_elements(self):
        return max(self.top * self.hidden, self.shared["hidden"] if self.shared else 0)

    def _run(self, h, out, ctx, accumulate):
        self._routed(h, out, ctx, accumulate)
        if self.shared:                                   # after the routed experts: `out` holds their sum by now
            T, Fs = h.shape[0], self.shared["hidden"]
            mid = ctx.ws.get("moe.shared.hidden", (T, Fs), h.dtype)
            self._gemm(ctx, h, self.ws_gate_up, mid, kernels.EPI_GATED, hidden=Fs)
            if self.ws_gate is None:
                self._gemm(ctx, mid, self.ws_down, out, kernels.EPI_ADD_F32)
            else:
                y = ctx.ws.get("moe.shared.y", (T, self.dim), torch.float32)
                self._gemm(ctx, mid, self.ws_down, y, kernels.EPI_STORE_F32)
                kernels.gated_add(y, h, self.ws_gate, out, True)
        return out

    def _routed(self, h, out, ctx, accumulate):
        T = h.shape[0]
        ws = ctx.ws
        ids = ws.get("moe.ids", (T, self.top), torch.int32)
        wts = ws.get("moe.weights", (T, self.top), torch.float32)
        logits = ws.get("moe.logits", (T, self.n_experts), torch.float32)        # products exact, sums in float32
        self._gemm(ctx, h, self.w_router, logits, kernels.EPI_STORE_F32)
        if self.corrected:
            kernels.moe_select_groups(logits, self.correction, ids, wts, self.groups, self.keep_groups, self.weight_scale,
                                      softmax=not self.sigmoid, group_max=self.group_max)
        else:
            kernels.moe_select(logits, ids, wts, self.renormalize, bias=self.b_router)
        if T >= GROUPED_MIN_ROWS and kernels.can_moe_grouped(self.dim, self.hidden, h.dtype, T * self.top, self.n_experts):
            return kernels.moe_grouped(h, self.w_gate, self.w_up, self.w_down, ids, wts, self.limit, self.alpha, ws.get,
                                       out, accumulate, up_shift=self.up_shift)
        mid = ws.get("moe.hidden", (T * self.top, self.hidden), h.dtype)
        kernels.moe_pair_gate_up(h, self.w_gate, self.w_up, ids, self.limit, self.alpha, mid, up_shift=self.up_shift)
        kernels.moe_pair_down(mid, self.w_down, ids, wts, out, accumulate)
        return out

    def forward(self, h, x, ctx):
        """Adds the result to x."""
        return self._run(h, x, ctx, True)

    def forward_to(self, h, y, ctx):
        """Writes the result to y (float32 [T, dim])."""
        return self._run(h, y, ctx, False)
