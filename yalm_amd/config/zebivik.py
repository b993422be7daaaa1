"""Typed configuration of the Zebivik design: a decoder whose layers are listed one by one in config.json, with a norm on either
side of every sublayer (x += c n(mixer(n(x))); x += c n(ff(n(x)))), the norm being an elementwise squash, tanh(alpha x) * w + b.
The token embedding passes that norm at once, the head is a matrix of its own, and its logits are capped.

config.json: `architecture` "Zebivik", `vocab`, `width`, `norm.eps`, `residual_mult`, `logit_softcap` (absent: no cap), and
`layers`, a list of
  {"type": "parallel", "mixer": {"left": {heads, kv_heads, dim, vdim, scale, rot?: {dims, base, scaling?: {factor, low, high,
     original}}}, "right": {heads, dim, vdim, decay: [a number a head]}, left_scale, right_scale}, "mlp": ...}
  {"type": "rglru", "mixer": {width, blocks, conv}, "mlp": ...}
  "mlp": null | {"kind": "dense", "ff", "limit"}
       | {"kind": "moe", "expert": {ff}, "router": {experts, top, scale, groups?: {count, keep}}, "shared"?: {ff}}.
Tensors: `embed`, `head`, and the norms `embed.norm`, `final.norm`, `l<i>.norm1`, `l<i>.norm1b`, `l<i>.norm2`, `l<i>.norm2b`, each
with `.b` and `.alpha` behind it;
  parallel: `l<i>.mix.left.{q,k,v,o}` with their biases `.b`, `l<i>.mix.left.g` [heads, width],
  `l<i>.mix.right.{q,k,v,g,o,norm}`;
  rglru: `l<i>.mix.{y,x,conv,ra,ri}` with their biases `.b`, `l<i>.mix.{lam,o}`;
  feed-forward: `l<i>.mlp.{gate,up,down}`, or `l<i>.mlp.{router,correction}` and `l<i>.mlp.{e<k>,shared}.{gate,up,down}`.

What the design fixes and this file therefore states: the attention turns element i of a head with element i + dims/2, sees
every earlier position and gates each head with one number; the linear attention's queries, keys and values are silus, and its
heads are normed together under a sigmoid gate; the recurrent block's rate of 8; the dense unit's 1.702 and its 1 beside the up
value; scores are a softmax over all experts, a correction counts in the choice and not in the weights, a group's score is its
largest choice score, and the chosen weights are brought to the sum router.scale; experts are silu(gate) * up."""
import copy
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from .llama import ConfigError
from .spec import LayerSpec, ModelSpec, PartSpec

MIXERS = ("parallel", "rglru")
UNIT_ALPHA, UNIT_SHIFT = 1.702, 1.0      # of the dense feed-forward's clamped unit
RATE = 8.0                       # of the recurrent block's decays
POSITIONS = 1 << 18              # the design names no longest sequence: the cache bounds it (and this, where nothing else does)


def _need(d, key, where):
    if not isinstance(d, dict) or key not in d or d[key] is None:
        raise ConfigError("config.json lacks the key %r in %s" % (key, where))
    return d[key]


def _ints(d, keys, where):
    return {k: int(_need(d, k, where)) for k in keys}


@dataclass(frozen=True)
class ZebivikConfig:
    vocab: int
    width: int
    eps: float
    residual_mult: float                             # of what a sublayer's outer norm adds to the stream
    logit_softcap: float = 0.0                       # 0: none
    layers: List[Dict[str, Any]] = field(default_factory=list)
    bos_token_id: Optional[int] = None
    eos_token_ids: List[int] = field(default_factory=list)

    ARCHITECTURES = ("Zebivik",)
    architecture = "Zebivik"

    # ------------------------------------------------------------------ reading
    @classmethod
    def from_dict(cls, d):
        arch = d.get("architecture") or (d.get("architectures") or [None])[0]
        if arch not in cls.ARCHITECTURES:
            raise ConfigError("architecture %r is not one of %s" % (arch, list(cls.ARCHITECTURES)))
        layers = _need(d, "layers", "config.json")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("`layers` must be a list with at least one layer")
        eos = d.get("eos_token_id")
        eos_ids = [] if eos is None else ([int(e) for e in eos] if isinstance(eos, (list, tuple)) else [int(eos)])
        cfg = cls(vocab=int(_need(d, "vocab", "config.json")), width=int(_need(d, "width", "config.json")),
                  eps=float(_need(_need(d, "norm", "config.json"), "eps", "norm")),
                  residual_mult=float(_need(d, "residual_mult", "config.json")), logit_softcap=float(d.get("logit_softcap") or 0.0),
                  layers=[cls._layer(i, l) for i, l in enumerate(layers)],
                  bos_token_id=None if d.get("bos_token_id") is None else int(d["bos_token_id"]), eos_token_ids=eos_ids)
        cfg.validate()
        return cfg

    @staticmethod
    def _left(m, where):
        out = _ints(m, ("heads",), where)
        out["kv_heads"] = int(m.get("kv_heads") or out["heads"])
        out["dim"] = int(_need(m, "dim", where))
        out["vdim"] = int(m.get("vdim") or out["dim"])
        out["scale"] = float(_need(m, "scale", where))
        if m.get("rot"):
            rot = {"dims": int(_need(m["rot"], "dims", where + ".rot")), "base": float(_need(m["rot"], "base", where + ".rot"))}
            if m["rot"].get("scaling"):
                rot["scaling"] = {k: float(_need(m["rot"]["scaling"], k, where + ".rot.scaling")) for k in ("factor", "low", "high", "original")}
            out["rot"] = rot
        return out

    @staticmethod
    def _right(m, where):
        out = _ints(m, ("heads", "dim"), where)
        out["vdim"] = int(m.get("vdim") or out["dim"])
        decay = _need(m, "decay", where)
        out["decay"] = [float(g) for g in decay] if isinstance(decay, (list, tuple)) else [float(decay)] * out["heads"]
        return out

    @classmethod
    def _layer(cls, i, l):
        where = "layer %d" % i
        kind = _need(l, "type", where)
        if kind not in MIXERS:
            raise ConfigError("%s: mixer type %r is not one of %s" % (where, kind, list(MIXERS)))
        m = _need(l, "mixer", where)
        if kind == "rglru":
            mixer = _ints(m, ("width", "blocks", "conv"), where)
        else:
            mixer = {"left": cls._left(_need(m, "left", where), where + ".left"), "right": cls._right(_need(m, "right", where), where + ".right")}
            mixer.update({k: float(_need(m, k, where)) for k in ("left_scale", "right_scale")})
        mlp = l.get("mlp")
        return {"type": kind, "mixer": mixer, "mlp": None if mlp is None else cls._mlp(mlp, where + ".mlp")}

    @staticmethod
    def _mlp(mlp, where):
        kind = _need(mlp, "kind", where)
        if kind == "dense":
            return {"kind": "dense", "ff": int(_need(mlp, "ff", where)), "limit": float(_need(mlp, "limit", where))}
        if kind != "moe":
            raise ConfigError("%s: feed-forward kind %r is neither 'dense' nor 'moe'" % (where, kind))
        ro = _need(mlp, "router", where)
        router = _ints(ro, ("experts", "top"), where + ".router")
        router["scale"] = float(_need(ro, "scale", where + ".router"))
        if ro.get("groups"):
            router["groups"] = _ints(ro["groups"], ("count", "keep"), where + ".router.groups")
        out = {"kind": "moe", "expert": _ints(_need(mlp, "expert", where), ("ff",), where + ".expert"), "router": router}
        if mlp.get("shared"):
            out["shared"] = _ints(mlp["shared"], ("ff",), where + ".shared")
        return out

    def validate(self):
        if self.vocab <= 0 or self.width <= 0 or not self.eps > 0 or self.logit_softcap < 0:
            raise ConfigError("vocab, width and norm.eps must be positive, logit_softcap not negative")
        for i, l in enumerate(self.layers):
            m, where = l["mixer"], "layer %d" % i
            if l["type"] == "rglru":
                if min(m["width"], m["blocks"], m["conv"]) <= 0 or m["width"] % m["blocks"]:
                    raise ConfigError("%s: width %d is no positive multiple of blocks %d, or conv %d is not positive"
                                      % (where, m["width"], m["blocks"], m["conv"]))
            else:
                left, right = m["left"], m["right"]
                if min(left[k] for k in ("heads", "kv_heads", "dim", "vdim")) <= 0 or min(right[k] for k in ("heads", "dim", "vdim")) <= 0:
                    raise ConfigError("%s: heads, kv_heads, dim and vdim must be positive" % where)
                if left["heads"] % left["kv_heads"]:
                    raise ConfigError("%s: heads %d is no multiple of kv_heads %d" % (where, left["heads"], left["kv_heads"]))
                rot = left.get("rot")
                if rot and (rot["dims"] < 0 or rot["dims"] % 2 or rot["dims"] > left["dim"] or not rot["base"] > 0):
                    raise ConfigError("%s: rot.dims must be even and at most dim, rot.base positive" % where)
                if rot and rot.get("scaling") and (not rot["scaling"]["factor"] > 0 or not rot["scaling"]["high"] >= rot["scaling"]["low"] > 0):
                    raise ConfigError("%s: rot.scaling needs a positive factor and high not below low" % where)
                if len(right["decay"]) != right["heads"] or not all(0.0 <= g <= 1.0 for g in right["decay"]):
                    raise ConfigError("%s: decay must hold a number from 0 to 1 for each of the %d heads" % (where, right["heads"]))
            if l["mlp"] is None:
                continue
            if l["mlp"]["kind"] == "dense":
                if l["mlp"]["ff"] <= 0 or not l["mlp"]["limit"] > 0:
                    raise ConfigError("%s: ff and limit must be positive" % where)
                continue
            r = l["mlp"]["router"]
            g = r.get("groups") or {"count": 1, "keep": 1}
            if l["mlp"]["expert"]["ff"] <= 0 or r["experts"] <= 0 or g["count"] <= 0 or r["experts"] % g["count"] \
                    or not 0 < g["keep"] <= g["count"] or not 0 < r["top"] <= g["keep"] * (r["experts"] // g["count"]) \
                    or l["mlp"].get("shared", {"ff": 1})["ff"] <= 0:
                raise ConfigError("%s: %d of %d experts in %d groups, %d of them kept, with ff %d do not go together"
                                  % (where, r["top"], r["experts"], g["count"], g["keep"], l["mlp"]["expert"]["ff"]))

    # ------------------------------------------------------------------ writing
    def to_dict(self):
        d = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
             "residual_mult": self.residual_mult, "layers": copy.deepcopy(self.layers)}
        if self.logit_softcap:
            d["logit_softcap"] = self.logit_softcap
        if self.bos_token_id is not None:
            d["bos_token_id"] = self.bos_token_id
        if self.eos_token_ids:
            d["eos_token_id"] = self.eos_token_ids[0] if len(self.eos_token_ids) == 1 else list(self.eos_token_ids)
        return d

    # ------------------------------------------------------------------ the model as data
    def _attention(self, m):
        position, rot = None, m.get("rot")
        if rot and rot["dims"]:
            params = {"head_dim": m["dim"], "rotary_dim": rot["dims"], "theta": rot["base"], "weight_rows": "half_split"}
            if rot.get("scaling"):
                sc = rot["scaling"]
                params["scaling"] = {"rope_type": "llama3", "factor": sc["factor"], "low_freq_factor": sc["low"],
                                     "high_freq_factor": sc["high"], "original_max_position_embeddings": sc["original"]}
            position = PartSpec("rope", params)
        return PartSpec("shaped_attention", {
            "n_heads": m["heads"], "n_kv_heads": m["kv_heads"], "key_dim": m["dim"], "value_dim": m["vdim"], "scale": m["scale"],
            "biases": True, "out_bias": True, "gate": "heads", "position": position,
            "tensors": {"q": "q", "k": "k", "v": "v", "out": "o", "q_bias": "q.b", "k_bias": "k.b", "v_bias": "v.b", "out_bias": "o.b",
                        "gate": "g"}}, prefix="left.")

    def _mixer(self, l):
        m = l["mixer"]
        if l["type"] == "rglru":
            return PartSpec("rglru", {"width": m["width"], "blocks": m["blocks"], "taps": m["conv"], "rate": RATE}, prefix="mix.")
        r = m["right"]
        recurrence = PartSpec("lightning", {"n_heads": r["heads"], "key_dim": r["dim"], "value_dim": r["vdim"], "decay": list(r["decay"]),
                                            "eps": self.eps}, prefix="right.")
        return PartSpec("side_by_side", {"left": self._attention(m["left"]), "right": recurrence,
                                         "scales": (m["left_scale"], m["right_scale"])}, prefix="mix.")

    def _feed_forward(self, mlp):
        if mlp["kind"] == "dense":
            return PartSpec("swiglu", {"hidden": mlp["ff"], "limit": mlp["limit"], "alpha": UNIT_ALPHA, "up_shift": UNIT_SHIFT,
                                       "tensors": {"gate": "gate", "up": "up", "down": "down"}}, prefix="mlp.")
        r = mlp["router"]
        groups = r.get("groups") or {"count": 1, "keep": 1}
        params = {"hidden": mlp["expert"]["ff"], "n_experts": r["experts"], "top": r["top"], "up_shift": 0.0, "scores": "softmax",
                  "renormalize": True, "groups": groups["count"], "keep_groups": groups["keep"], "group_score": "max",
                  "weight_scale": r["scale"], "expert_prefix": "e%d.", "tensors": {"correction": "correction"}}
        if mlp.get("shared"):
            params["shared"] = {"hidden": mlp["shared"]["ff"], "prefix": "shared."}
        return PartSpec("moe", params, prefix="mlp.")

    def to_spec(self):
        def norm(tensor, **kw):
            return PartSpec("dynamic_tanh", dict(kw, tensor=tensor))
        layers = []
        for i, l in enumerate(self.layers):
            members = {"mixer_norm": norm("norm1"), "mixer": self._mixer(l), "mixer_out_norm": norm("norm1b", result_scale=self.residual_mult)}
            if l["mlp"] is not None:
                members.update({"feed_forward_norm": norm("norm2"), "feed_forward": self._feed_forward(l["mlp"]),
                                "feed_forward_out_norm": norm("norm2b", result_scale=self.residual_mult)})
            layers.append(LayerSpec("sandwich_residual", parts=members, prefix="l%d." % i))
        return ModelSpec(
            architecture=self.architecture, dim=self.width, vocab_size=self.vocab, max_positions=POSITIONS,
            embedding=PartSpec("token_embedding", {"vocab_size": self.vocab, "tensor": "embed", "norm": norm("embed.norm")}),
            layers=layers, final_norm=norm("final.norm"),
            head=PartSpec("lm_head", {"vocab_size": self.vocab, "tied": False, "tensor": "head", "softcap": self.logit_softcap}),
            bos_token_id=self.bos_token_id, eos_token_ids=list(self.eos_token_ids))
