"""A plain, slow implementation of the Gemepel design in float64 torch on the CPU: one function per mechanism,
written from the design's equations and sharing nothing with yalm_amd.  The tests hold the library against it.

The design: a decoder that norms the SUM of stream and sublayer,
    x <- LN1(a x + mixer(x)),   x <- LN2(a x + ff(x)),      LN(x) = (x - mean) / sqrt(var + eps) * w + b
(the sublayers read x itself; a is one number of the model).  Tokens are embedded by their own row, scaled, plus a
row of a second table that the pair (previous token, token) hashes to.  Mixers: latent attention whose queries
pass a latent vector of their own, or a gated linear attention (a recurrence with a decay per key channel made by a
low-rank product).  Feed-forwards: a mixture of two-matrix experts with squared-relu units, chosen by sigmoid scores
plus a correction inside the best groups of experts.

`weights` is a dictionary name -> tensor with the names of a model folder ('l3.mix.q', ...).  `memory`, where a
function takes one, is what is kept of earlier tokens of ONE sequence: a dictionary the functions fill and read,
so that a text can be fed in pieces."""
import math

import torch

F64 = torch.float64


def W(w, name):
    return w[name].to(F64)


def rms_norm(x, weight, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * weight


def layer_norm(x, weight, bias, eps):
    d = x - x.mean(dim=-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(dim=-1, keepdim=True) + eps) * weight + bias


def norm(x, w, name, eps):
    return layer_norm(x, W(w, name), W(w, name + ".b"), eps)


def silu(z):
    return z * torch.sigmoid(z)


# ------------------------------------------------------------------------------------------ embedding
def pair_row(previous, token, bigram):
    """The row of the pair table for a token behind `previous` (None: the sequence's first token)."""
    if previous is None:
        return int(bigram["buckets"])
    return (int(previous) * int(bigram["mul_prev"]) + int(token) * int(bigram["mul_cur"])) % int(bigram["buckets"])


def embed(tokens, embedding, w, memory):
    x = W(w, "embed")[torch.as_tensor(tokens, dtype=torch.long)] * float(embedding["scale"])
    if embedding.get("bigram"):
        rows = []
        for t in tokens:
            rows.append(pair_row(memory.get("token"), t, embedding["bigram"]))
            memory["token"] = int(t)
        x = x + W(w, "bigram")[torch.tensor(rows, dtype=torch.long)]
    return x


# ------------------------------------------------------------------------------------------ latent attention
def rotate_pairs(v, positions, dims, base):
    """The first `dims` elements of the last axis of v [T, ..., n], pair (2i, 2i + 1) turned by the angle
    position * base^(-2i / dims); the others pass."""
    if not dims:
        return v
    f = torch.tensor([float(base) ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F64)
    a = (positions.to(F64)[:, None] * f).reshape([v.shape[0]] + [1] * (v.dim() - 2) + [dims // 2])
    out = v.clone()
    u, z = v[..., 0:dims:2], v[..., 1:dims:2]
    out[..., 0:dims:2] = u * torch.cos(a) - z * torch.sin(a)
    out[..., 1:dims:2] = z * torch.cos(a) + u * torch.sin(a)
    return out


def latent_queries(h, positions, m, w, p, eps):
    """[T, heads, dim] unrotated and [T, heads, rot_dim] rotated, through the queries' latent vector."""
    H, d, r = int(m["heads"]), int(m["dim"]), int(m["rot_dim"])
    c = rms_norm(h @ W(w, p + "dq").T, W(w, p + "dq.norm"), eps)
    q = (c @ W(w, p + "uq").T).reshape(h.shape[0], H, d + r)
    return q[..., :d], rotate_pairs(q[..., d:], positions, int(m["rot"]["dims"]), m["rot"]["base"])


def latent_keys(h, positions, m, w, p, eps):
    """What is remembered of the tokens: the latent vectors [T, kv_rank] and the shared rotated key part."""
    R = int(m["kv_rank"])
    z = h @ W(w, p + "dkv").T
    c = rms_norm(z[:, :R], W(w, p + "dkv.norm"), eps)
    return c, rotate_pairs(z[:, R:], positions, int(m["rot"]["dims"]), m["rot"]["base"])


def latent_attention(h, positions, m, w, p, eps, kept):
    """kept = (c, rotated keys) of positions 0 .. (the queries' own among them)."""
    H, d, vd = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q, q_rot = latent_queries(h, positions, m, w, p, eps)
    c, k_rot = kept
    S = c.shape[0]
    k = (c @ W(w, p + "uk").T).reshape(S, H, d)
    v = (c @ W(w, p + "uv").T).reshape(S, H, vd)
    score = (torch.einsum("thd,shd->hts", q, k) + torch.einsum("thd,sd->hts", q_rot, k_rot)) * float(m["scale"])
    later = torch.arange(S)[None, :] > positions[:, None]
    prob = torch.softmax(score.masked_fill(later[None], float("-inf")), dim=-1)
    return torch.einsum("hts,shv->thv", prob, v).reshape(h.shape[0], H * vd) @ W(w, p + "o").T


# ------------------------------------------------------------------------------------------ gated linear attention
def decays(h, m, w, p):
    """[T, heads, dim] in (0, 1): sigmoid(z)^(1 / tau) with z a low-rank product plus a bias."""
    z = (h @ W(w, p + "a1").T) @ W(w, p + "a2").T + W(w, p + "a2.b")
    return torch.sigmoid(z).pow(1.0 / float(m["tau"])).reshape(h.shape[0], int(m["heads"]), int(m["dim"]))


def gla_scan(q, k, v, a, state):
    """One head: q, k, a [T, d], v [T, dv], state [d, dv] -> ([T, dv], state)."""
    out = []
    for t in range(q.shape[0]):
        state = a[t][:, None] * state + k[t][:, None] * v[t][None, :]
        out.append(state.T @ q[t])
    return torch.stack(out), state


def gla(h, m, w, p, eps, memory, faint_out=None):
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    T = h.shape[0]
    q = (h @ W(w, p + "q").T).reshape(T, H, d) * d ** -0.5
    k = (h @ W(w, p + "k").T).reshape(T, H, d)
    v = (h @ W(w, p + "v").T).reshape(T, H, dv)
    a = decays(h, m, w, p)
    state = memory.get("state")
    state = torch.zeros((H, d, dv), dtype=F64) if state is None else state
    outs, states = zip(*[gla_scan(q[:, i], k[:, i], v[:, i], a[:, i], state[i]) for i in range(H)])
    memory["state"] = torch.stack(states)
    if faint_out is not None:                      # a head's read-out beside the layer's median: its norm divides by it
        size = torch.stack(outs, dim=1).pow(2).mean(dim=-1).sqrt()
        faint_out.append((size / size.median().clamp_min(1e-30)).min(dim=-1).values)
    o = rms_norm(torch.stack(outs, dim=1), W(w, p + "norm"), eps).reshape(T, H * dv)
    return (o * silu(h @ W(w, p + "g").T)) @ W(w, p + "o").T


# ------------------------------------------------------------------------------------------ mixture of experts
def choice_scores(h, router, w, p):
    """(scores [T, experts], choice scores with the experts outside the kept groups at minus infinity)."""
    s = torch.sigmoid(h @ W(w, p + "router").T)
    c = s + W(w, p + "correction")
    g = router.get("groups")
    if g:
        T, n = c.shape[0], int(g["count"])
        grouped = c.reshape(T, n, -1)
        score = torch.topk(grouped, min(2, grouped.shape[-1]), dim=-1).values.sum(dim=-1)
        kept = torch.zeros((T, n), dtype=torch.bool)
        kept.scatter_(1, torch.topk(score, int(g["keep"]), dim=-1).indices, True)
        c = grouped.masked_fill(~kept[..., None], float("-inf")).reshape(T, -1)
    return s, c


def route(h, router, w, p):
    """(chosen experts [T, top] by falling choice score, their weights)."""
    s, c = choice_scores(h, router, w, p)
    chosen = torch.topk(c, int(router["top"]), dim=-1).indices
    weight = torch.gather(s, 1, chosen)
    return chosen, weight / (weight.sum(dim=-1, keepdim=True) + 1e-20) * float(router["scale"])


def route_margin(h, router, w, p):
    """How decided a token's choice is: the smallest gap that, closed, would choose otherwise (between the last
    kept and the first dropped group's scores, and between the last chosen and the first passed-over expert's choice
    scores), relative to the spread of the choice scores.  A computation in fewer bits may choose otherwise where
    this is small."""
    s = torch.sigmoid(h @ W(w, p + "router").T) + W(w, p + "correction")
    _, c = choice_scores(h, router, w, p)
    T, top = c.shape[0], int(router["top"])
    spread = s.std(dim=-1, unbiased=False).clamp_min(1e-6)
    gap = torch.full((T,), float("inf"), dtype=F64)
    if top < c.shape[1]:
        best = torch.topk(c, top + 1, dim=-1).values
        gap = torch.minimum(gap, best[:, top - 1] - best[:, top])
    g = router.get("groups")
    if g and int(g["keep"]) < int(g["count"]):
        grouped = s.reshape(T, int(g["count"]), -1)
        score = torch.topk(grouped, min(2, grouped.shape[-1]), dim=-1).values.sum(dim=-1)
        best = torch.topk(score, int(g["keep"]) + 1, dim=-1).values
        gap = torch.minimum(gap, best[:, -2] - best[:, -1])
    return gap / spread


def expert(h, w, p):
    return torch.relu(h @ W(w, p + "up").T) ** 2 @ W(w, p + "down").T


def moe(h, mlp, w, p):
    chosen, weight = route(h, mlp["router"], w, p)
    rows = []
    for t in range(h.shape[0]):
        rows.append(sum(weight[t, i] * expert(h[t:t + 1], w, "%se%d." % (p, int(chosen[t, i])))[0]
                        for i in range(chosen.shape[1])))
    return torch.stack(rows)


# ------------------------------------------------------------------------------------------ the model
def mixer(i, layer, x, positions, w, eps, memory, faint_out=None):
    m, p = layer["mixer"], "l%d.mix." % i
    if layer["type"] == "gla":
        return gla(x, m, w, p, eps, memory.setdefault(i, {}), faint_out)
    src = m.get("kv_from")
    if src is None:
        made = latent_keys(x, positions, m, w, p, eps)
        mine = memory.setdefault(i, {})
        mine["kept"] = made if "kept" not in mine else tuple(torch.cat(z) for z in zip(mine["kept"], made))
    return latent_attention(x, positions, m, w, p, eps, memory[i if src is None else int(src)]["kept"])


def forward(config, w, tokens, memory=None, start=0, layers_out=None, margins_out=None, faint_out=None):
    """Logits [T, vocab] of one sequence's tokens at positions start.. .  memory: {} at the sequence's start, handed
    in again to go on.  layers_out: a list that receives the residual stream after every layer; margins_out: one that
    receives route_margin [T] of every feed-forward; faint_out: one that receives, for every recurrence, how small the
    smallest head's read-out is beside the layer's median [T]."""
    eps, alpha = float(config["norm"]["eps"]), float(config["postln_alpha"])
    memory = {} if memory is None else memory
    tokens = [int(t) for t in tokens]
    positions = torch.arange(start, start + len(tokens))
    x = embed(tokens, config["embedding"], w, memory)
    for i, layer in enumerate(config["layers"]):
        p = "l%d." % i
        x = norm(alpha * x + mixer(i, layer, x, positions, w, eps, memory, faint_out), w, p + "norm1", eps)
        if layer.get("mlp"):
            if margins_out is not None:
                margins_out.append(route_margin(x, layer["mlp"]["router"], w, p + "mlp."))
            x = norm(alpha * x + moe(x, layer["mlp"], w, p + "mlp."), w, p + "norm2", eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return norm(x, w, "final.norm", eps) @ W(w, "head").T
