"""A plain, slow implementation of the Zebivik design in float64 torch on the CPU: one function per mechanism,
written from the design's equations and sharing nothing with yalm_amd.  The tests hold the library against it.

The design: a decoder with a norm on either side of every sublayer,
    x <- x + c n1b(mixer(n1(x))),   x <- x + c n2b(ff(n2(x))),      n(x) = tanh(alpha x) * w + b
(n forms no mean; c is one number of the model).  Mixers: an attention with one gate a head side by side with a
linear attention of fixed decays (a weighted sum of both results), or Griffin's recurrent block around a gated linear
recurrence.  Feed-forwards: a dense clamped gated unit, or a mixture of experts chosen inside the best groups by softmax
scores plus a correction, beside a shared expert.  The logits are capped.

`weights` is a dictionary name -> tensor with the names of a model folder ('l3.mix.y', ...).  `memory`, where a
function takes one, is what is kept of earlier tokens of ONE sequence: a dictionary the functions fill and read,
so that a text can be fed in pieces."""
import math

import torch

F64 = torch.float64


def W(w, name):
    return w[name].to(F64)


def rms_norm(x, weight, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * weight


def norm(x, w, name):
    """The model's norm: an elementwise squash."""
    return torch.tanh(W(w, name + ".alpha") * x) * W(w, name) + W(w, name + ".b")


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def linear(h, w, name):
    out = h @ W(w, name).T
    return out + W(w, name + ".b") if name + ".b" in w else out


# ------------------------------------------------------------------------------------------ attention
def frequencies(rot):
    """base^(-2i / dims), slowed down for the long wavelengths as rot.scaling says."""
    out = []
    sc = rot.get("scaling")
    for i in range(int(rot["dims"]) // 2):
        f = float(rot["base"]) ** (-2.0 * i / int(rot["dims"]))
        if sc:
            turns = float(sc["original"]) * f / (2.0 * math.pi)             # within the original length
            low, high, factor = float(sc["low"]), float(sc["high"]), float(sc["factor"])
            if turns < low:
                f = f / factor
            elif turns <= high:
                s = (turns - low) / (high - low)
                f = (1.0 - s) * f / factor + s * f
        out.append(f)
    return torch.tensor(out, dtype=F64)


def rotate(v, positions, rot):
    """v [T, heads, n]: element i turned together with element i + dims/2, for the first `dims` elements."""
    if not rot or not int(rot["dims"]):
        return v
    half = int(rot["dims"]) // 2
    a = (positions.to(F64)[:, None] * frequencies(rot))[:, None, :]
    u, z = v[..., :half], v[..., half:2 * half]
    return torch.cat([u * torch.cos(a) - z * torch.sin(a), z * torch.cos(a) + u * torch.sin(a), v[..., 2 * half:]], dim=-1)


def attend(q, k, v, positions, scale):
    """q [T, H, d] at `positions`, k [S, G, d] and v [S, G, dv] of the positions 0 .. S - 1 -> [T, H, dv]."""
    H, G = q.shape[1], k.shape[1]
    k, v = k.repeat_interleave(H // G, dim=1), v.repeat_interleave(H // G, dim=1)
    score = torch.einsum("thd,shd->hts", q, k) * scale
    later = torch.arange(k.shape[0])[None, :] > positions[:, None]
    prob = torch.softmax(score.masked_fill(later[None], float("-inf")), dim=-1)
    return torch.einsum("hts,shv->thv", prob, v)


def attention(h, positions, m, w, p, memory):
    T, H, G, d, dv = h.shape[0], int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = rotate(linear(h, w, p + "q").reshape(T, H, d), positions, m.get("rot"))
    k = rotate(linear(h, w, p + "k").reshape(T, G, d), positions, m.get("rot"))
    v = linear(h, w, p + "v").reshape(T, G, dv)
    if "k" in memory:
        k, v = torch.cat([memory["k"], k]), torch.cat([memory["v"], v])
    memory["k"], memory["v"] = k, v
    o = attend(q, k, v, positions, float(m["scale"])) * torch.sigmoid(h @ W(w, p + "g").T)[..., None]
    return linear(o.reshape(T, H * dv), w, p + "o")


# ------------------------------------------------------------------------------------------ linear attention, fixed decays
def decay_scan(q, k, v, decay, state):
    """One head: q, k [T, d], v [T, dv], a number `decay`, state [d, dv] -> ([T, dv], state)."""
    out = []
    for t in range(q.shape[0]):
        state = decay * state + k[t][:, None] * v[t][None, :]
        out.append(state.T @ q[t])
    return torch.stack(out), state


def lightning(h, m, w, p, eps, memory, faint_out=None):
    T, H, d, dv = h.shape[0], int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q, k = (silu(h @ W(w, p + n).T).reshape(T, H, d) for n in "qk")
    v = silu(h @ W(w, p + "v").T).reshape(T, H, dv)
    state = memory.get("state")
    state = torch.zeros((H, d, dv), dtype=F64) if state is None else state
    outs, states = zip(*[decay_scan(q[:, i], k[:, i], v[:, i], float(m["decay"][i]), state[i]) for i in range(H)])
    memory["state"] = torch.stack(states)
    o = torch.stack(outs, dim=1).reshape(T, H * dv)
    if faint_out is not None:                      # a row that is small beside the others: its norm divides by it
        size = o.pow(2).mean(dim=-1).sqrt()
        faint_out.append(size / size.median().clamp_min(1e-30))
    return (rms_norm(o, W(w, p + "norm"), eps) * torch.sigmoid(h @ W(w, p + "g").T)) @ W(w, p + "o").T


def parallel(h, positions, m, w, p, eps, memory, faint_out=None):
    left = attention(h, positions, m["left"], w, p + "left.", memory.setdefault("left", {}))
    right = lightning(h, m["right"], w, p + "right.", eps, memory.setdefault("right", {}), faint_out)
    return float(m["left_scale"]) * left + float(m["right_scale"]) * right


# ------------------------------------------------------------------------------------------ the recurrent block
def causal_conv(x, taps_w, bias, memory):
    """x [T, C]: sum over j of taps_w[:, j] times the input j - (taps - 1) tokens away, zeros before the text."""
    taps = taps_w.shape[1]
    past = memory.get("inputs")
    past = torch.zeros((taps - 1, x.shape[1]), dtype=F64) if past is None else past
    seen = torch.cat([past, x])
    memory["inputs"] = seen[seen.shape[0] - (taps - 1):]
    return torch.stack([(seen[t:t + taps].T * taps_w).sum(dim=1) for t in range(x.shape[0])]) + bias


def block_gate(u, mats, bias):
    """sigmoid of a product in every block: u [T, blocks * n], mats [blocks, n, n] as [out, in], bias [blocks, n]."""
    nb, n = bias.shape
    return torch.sigmoid(torch.einsum("tbi,boi->tbo", u.reshape(-1, nb, n), mats) + bias).reshape(u.shape)


def lru_scan(u, r, i, lam, state):
    """S <- a S + sqrt(1 - a^2) i u with a = exp(-8 r softplus(lam)); u, r, i [T, C] -> ([T, C], S [C])."""
    log_a = -8.0 * r * torch.log1p(torch.exp(-lam.abs())) - 8.0 * r * lam.clamp_min(0.0)
    out = []
    for t in range(u.shape[0]):
        state = torch.exp(log_a[t]) * state + torch.sqrt(-torch.expm1(2.0 * log_a[t])) * i[t] * u[t]
        out.append(state)
    return torch.stack(out), state


def rglru(h, m, w, p, memory):
    y = gelu_tanh(linear(h, w, p + "y"))
    u = causal_conv(linear(h, w, p + "x"), W(w, p + "conv"), W(w, p + "conv.b"), memory)
    r, i = (block_gate(u, W(w, p + n), W(w, p + n + ".b")) for n in ("ra", "ri"))
    state = memory.get("state")
    state = torch.zeros(u.shape[1], dtype=F64) if state is None else state
    s, memory["state"] = lru_scan(u, r, i, W(w, p + "lam"), state)
    return (s * y) @ W(w, p + "o").T


# ------------------------------------------------------------------------------------------ feed-forwards
def clamped_unit(h, limit, w, p):
    g = (h @ W(w, p + "gate").T).clamp(max=limit)
    u = (h @ W(w, p + "up").T).clamp(-limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ W(w, p + "down").T


def expert(h, w, p):
    return (silu(h @ W(w, p + "gate").T) * (h @ W(w, p + "up").T)) @ W(w, p + "down").T


def group_scores(c, n):
    """The largest choice score of each of n equal groups of neighbours."""
    return c.reshape(c.shape[0], n, -1).max(dim=-1).values


def choice_scores(h, router, w, p):
    """(scores [T, experts], choice scores with the experts outside the kept groups at minus infinity)."""
    s = torch.softmax(h @ W(w, p + "router").T, dim=-1)
    c = s + W(w, p + "correction")
    g = router.get("groups")
    if g:
        n, T = int(g["count"]), c.shape[0]
        kept = torch.zeros((T, n), dtype=torch.bool)
        kept.scatter_(1, torch.topk(group_scores(c, n), int(g["keep"]), dim=-1).indices, True)
        c = c.reshape(T, n, -1).masked_fill(~kept[..., None], float("-inf")).reshape(T, -1)
    return s, c


def route(h, router, w, p):
    """(chosen experts [T, top] by falling choice score, their weights)."""
    s, c = choice_scores(h, router, w, p)
    chosen = torch.topk(c, int(router["top"]), dim=-1).indices
    weight = torch.gather(s, 1, chosen)
    return chosen, weight / (weight.sum(dim=-1, keepdim=True) + 1e-20) * float(router["scale"])


def route_margin(h, router, w, p):
    """How decided a token's choice is: the smallest gap that, closed, would choose otherwise, relative to the spread of
    the choice scores.  A computation in fewer bits may choose otherwise where this is small."""
    s, c = choice_scores(h, router, w, p)
    raw = s + W(w, p + "correction")
    T, top = c.shape[0], int(router["top"])
    spread = raw.std(dim=-1, unbiased=False).clamp_min(1e-6)
    gap = torch.full((T,), float("inf"), dtype=F64)
    if top < c.shape[1]:
        best = torch.topk(c, top + 1, dim=-1).values
        gap = torch.minimum(gap, best[:, top - 1] - best[:, top])
    g = router.get("groups")
    if g and int(g["keep"]) < int(g["count"]):
        best = torch.topk(group_scores(raw, int(g["count"])), int(g["keep"]) + 1, dim=-1).values
        gap = torch.minimum(gap, best[:, -2] - best[:, -1])
    return gap / spread


def moe(h, mlp, w, p):
    chosen, weight = route(h, mlp["router"], w, p)
    rows = []
    for t in range(h.shape[0]):
        rows.append(sum(weight[t, i] * expert(h[t:t + 1], w, "%se%d." % (p, int(chosen[t, i])))[0]
                        for i in range(chosen.shape[1])))
    out = torch.stack(rows)
    return out + expert(h, w, p + "shared.") if mlp.get("shared") else out


# ------------------------------------------------------------------------------------------ the model
def mixer(i, layer, h, positions, w, eps, memory, faint_out=None):
    m, p, mine = layer["mixer"], "l%d.mix." % i, memory.setdefault(i, {})
    if layer["type"] == "rglru":
        return rglru(h, m, w, p, mine)
    return parallel(h, positions, m, w, p, eps, mine, faint_out)


def forward(config, w, tokens, memory=None, start=0, layers_out=None, margins_out=None, faint_out=None):
    """Logits [T, vocab] of one sequence's tokens at positions start.. .  memory: {} at the sequence's start, handed
    in again to go on.  layers_out: a list that receives the residual stream after every layer; margins_out: one that
    receives route_margin [T] of every mixture; faint_out: one that receives, for every linear attention, how small a
    token's read-out is beside the layer's median [T]."""
    eps, c = float(config["norm"]["eps"]), float(config["residual_mult"])
    memory = {} if memory is None else memory
    tokens = torch.as_tensor([int(t) for t in tokens], dtype=torch.long)
    positions = torch.arange(start, start + len(tokens))
    x = norm(W(w, "embed")[tokens], w, "embed.norm")
    for i, layer in enumerate(config["layers"]):
        p, mlp = "l%d." % i, layer.get("mlp")
        x = x + c * norm(mixer(i, layer, norm(x, w, p + "norm1"), positions, w, eps, memory, faint_out), w, p + "norm1b")
        if mlp:
            h = norm(x, w, p + "norm2")
            if mlp["kind"] == "moe":
                if margins_out is not None:
                    margins_out.append(route_margin(h, mlp["router"], w, p + "mlp."))
                y = moe(h, mlp, w, p + "mlp.")
            else:
                y = clamped_unit(h, float(mlp["limit"]), w, p + "mlp.")
            x = x + c * norm(y, w, p + "norm2b")
        if layers_out is not None:
            layers_out.append(x.clone())
    logits = norm(x, w, "final.norm") @ W(w, "head").T
    cap = config.get("logit_softcap")
    return float(cap) * torch.tanh(logits / float(cap)) if cap else logits
