"""Typed configuration of the Gemepel design: a decoder whose layers are listed one by one in config.json and norm the sum of
stream and sublayer (x <- LN(alpha x + mixer(x)); x <- LN(alpha x + ff(x))), with a latent attention or a gated linear
attention as mixer and a mixture of experts as feed-forward (or none).  A token's embedding is its own row, scaled, plus
the row of a second table that the pair of the previous token and this one hashes to.

config.json: `architecture` "Gemepel", `vocab`, `width`, `norm.eps`, `postln_alpha`, `embedding` {scale, bigram?: {buckets,
mul_prev, mul_cur}}, and `layers`, a list of
  {"type": "latent_attention",
   "mixer": {heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, rot: {base, dims}, kv_from?: j}, "mlp": ...}
  {"type": "gla", "mixer": {heads, dim, vdim, tau, decay_rank?}, "mlp": ...}
  "mlp": null | {"kind": "moe", "expert": {ff}, "router": {experts, top, scale, groups?: {count, keep}}}.
Tensors: `embed`, `bigram` [buckets + 1, width], `head`, `final.norm` and for layer i `l<i>.norm1`, `l<i>.norm2`, each norm with
its bias behind `.b`;
  latent_attention: `l<i>.mix.{dq,dq.norm,uq,dkv,dkv.norm,uk,uv,o}` (no `dkv` with kv_from);
  gla: `l<i>.mix.{q,k,v,g,a1,a2,a2.b,norm,o}`;
  feed-forward: `l<i>.mlp.{router,correction,e<k>.up,e<k>.down}`.
The inner size of a gla mixer's low-rank product (`a1`/`a2`) is the tensors' own: a folder's configuration takes it from the
shape of `a1` (`with_tensor_shapes`); `decay_rank` names it where there is no folder yet (random models, and `to_dict`
writes it).  The sizes of the queries' and keys' latent vectors are config.json's.

What the design fixes and this file therefore states: the rotation pairs neighbouring elements (2i, 2i + 1); every query
sees every earlier position; the gla queries' scale dim^(-1/2); experts of two matrices with squared-relu units; scores
are sigmoids, a correction counts in the choice and not in the weights, and the chosen weights are brought to the sum
router.scale; the norms on latent vectors and heads are RMS norms, all others layer norms with bias, all with the one eps."""
import copy
from dataclasses import dataclass, field, replace
from typing import Any, Dict, List, Optional

from .llama import ConfigError
from .spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry

MIXERS = ("latent_attention", "gla")
POSITIONS = 1 << 18              # the design names no longest sequence: the cache bounds it (and this, where nothing else does)


def _need(d, key, where):
    if not isinstance(d, dict) or key not in d or d[key] is None:
        raise ConfigError("config.json lacks the key %r in %s" % (key, where))
    return d[key]


@dataclass(frozen=True)
class GemepelConfig:
    vocab: int
    width: int
    eps: float
    alpha: float                                   # of the stream in the sum that a layer norms
    embedding_scale: float
    bigram: Optional[Dict[str, int]] = None
    layers: List[Dict[str, Any]] = field(default_factory=list)
    bos_token_id: Optional[int] = None
    eos_token_ids: List[int] = field(default_factory=list)

    ARCHITECTURES = ("Gemepel",)
    architecture = "Gemepel"

    # ------------------------------------------------------------------ reading
    @classmethod
    def from_dict(cls, d):
        arch = d.get("architecture") or (d.get("architectures") or [None])[0]
        if arch not in cls.ARCHITECTURES:
            raise ConfigError("architecture %r is not one of %s" % (arch, list(cls.ARCHITECTURES)))
        layers = _need(d, "layers", "config.json")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("`layers` must be a list with at least one layer")
        emb = _need(d, "embedding", "config.json")
        bigram = None
        if emb.get("bigram"):
            bigram = {k: int(_need(emb["bigram"], k, "embedding.bigram")) for k in ("buckets", "mul_prev", "mul_cur")}
        eos = d.get("eos_token_id")
        eos_ids = [] if eos is None else ([int(e) for e in eos] if isinstance(eos, (list, tuple)) else [int(eos)])
        cfg = cls(vocab=int(_need(d, "vocab", "config.json")), width=int(_need(d, "width", "config.json")),
                  eps=float(_need(_need(d, "norm", "config.json"), "eps", "norm")),
                  alpha=float(_need(d, "postln_alpha", "config.json")), embedding_scale=float(_need(emb, "scale", "embedding")),
                  bigram=bigram, layers=[cls._layer(i, l) for i, l in enumerate(layers)],
                  bos_token_id=None if d.get("bos_token_id") is None else int(d["bos_token_id"]), eos_token_ids=eos_ids)
        cfg.validate()
        return cfg

    @staticmethod
    def _layer(i, l):
        where = "layer %d" % i
        kind = _need(l, "type", where)
        if kind not in MIXERS:
            raise ConfigError("%s: mixer type %r is not one of %s" % (where, kind, list(MIXERS)))
        m = _need(l, "mixer", where)
        mixer = {k: int(_need(m, k, where)) for k in ("heads", "dim", "vdim")}
        if kind == "gla":
            mixer["tau"] = float(_need(m, "tau", where))
            if m.get("decay_rank") is not None:
                mixer["decay_rank"] = int(m["decay_rank"])
        else:
            mixer.update({k: int(_need(m, k, where)) for k in ("rot_dim", "q_rank", "kv_rank")})
            rot = _need(m, "rot", where + ".mixer")
            mixer["scale"] = float(_need(m, "scale", where))
            mixer["rot"] = {"base": float(_need(rot, "base", where + ".rot")), "dims": int(_need(rot, "dims", where + ".rot"))}
            if m.get("kv_from") is not None:
                mixer["kv_from"] = int(m["kv_from"])
        mlp = l.get("mlp")
        if mlp is not None:
            if _need(mlp, "kind", where + ".mlp") != "moe":
                raise ConfigError("%s: feed-forward kind %r is not 'moe'" % (where, mlp["kind"]))
            ro = _need(mlp, "router", where + ".mlp")
            router = {k: int(_need(ro, k, where + ".router")) for k in ("experts", "top")}
            router["scale"] = float(_need(ro, "scale", where + ".router"))
            if ro.get("groups"):
                router["groups"] = {k: int(_need(ro["groups"], k, where + ".router.groups")) for k in ("count", "keep")}
            mlp = {"kind": "moe", "expert": {"ff": int(_need(_need(mlp, "expert", where + ".mlp"), "ff", where + ".expert"))},
                   "router": router}
        return {"type": kind, "mixer": mixer, "mlp": mlp}

    def validate(self):
        if self.vocab <= 0 or self.width <= 0 or not self.eps > 0:
            raise ConfigError("vocab, width and norm.eps must be positive")
        if self.bigram is not None and self.bigram["buckets"] <= 0:
            raise ConfigError("embedding.bigram.buckets must be positive")
        for i, l in enumerate(self.layers):
            m, where = l["mixer"], "layer %d" % i
            for k in ("heads", "dim", "vdim"):
                if m[k] <= 0:
                    raise ConfigError("%s: %s must be positive" % (where, k))
            if l["type"] == "gla":
                if not m["tau"] > 0 or m.get("decay_rank", 1) <= 0:
                    raise ConfigError("%s: tau and decay_rank must be positive" % where)
            else:
                dims = m["rot"]["dims"]
                if m["q_rank"] <= 0 or m["kv_rank"] <= 0:
                    raise ConfigError("%s: q_rank and kv_rank must be positive" % where)
                if m["rot_dim"] < 0 or m["rot_dim"] % 2 or dims % 2 or not 0 <= dims <= m["rot_dim"]:
                    raise ConfigError("%s: rot_dim %d and rot.dims %d must be even, dims at most rot_dim" % (where, m["rot_dim"], dims))
                j = m.get("kv_from")
                if j is not None:
                    if not 0 <= j < i or self.layers[j]["type"] != "latent_attention" \
                            or self.layers[j]["mixer"].get("kv_from") is not None:
                        raise ConfigError("%s: kv_from %r must name an earlier latent attention that makes its own keys" % (where, j))
                    if any(self.layers[j]["mixer"][k] != m[k] for k in ("kv_rank", "rot_dim", "rot")):
                        raise ConfigError("%s: layer %d, whose keys it uses, differs in kv_rank, rot_dim or rotation" % (where, j))
            if l["mlp"]:
                r, n = l["mlp"]["router"], 1
                keep = 1
                if r.get("groups"):
                    n, keep = r["groups"]["count"], r["groups"]["keep"]
                if l["mlp"]["expert"]["ff"] <= 0 or r["experts"] <= 0 or n <= 0 or r["experts"] % n or not 0 < keep <= n \
                        or not 0 < r["top"] <= keep * (r["experts"] // n):
                    raise ConfigError("%s: %d of %d experts in %d groups, %d of them kept, with ff %d do not go together"
                                      % (where, r["top"], r["experts"], n, keep, l["mlp"]["expert"]["ff"]))

    def with_tensor_shapes(self, shape_of):
        """The configuration with the sizes that only a folder's tensors give: `shape_of(name)` is a tensor's shape or
        None.  A gla mixer's decay_rank is the rows of its `a1`."""
        layers = copy.deepcopy(self.layers)
        for i, l in enumerate(layers):
            shape = shape_of("l%d.mix.a1" % i) if l["type"] == "gla" else None
            if shape is not None and len(shape) == 2:
                l["mixer"]["decay_rank"] = int(shape[0])
        cfg = replace(self, layers=layers)
        cfg.validate()
        return cfg

    # ------------------------------------------------------------------ writing
    def to_dict(self):
        embedding = {"scale": self.embedding_scale}
        if self.bigram is not None:
            embedding["bigram"] = dict(self.bigram)
        d = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
             "postln_alpha": self.alpha, "embedding": embedding, "layers": copy.deepcopy(self.layers)}
        if self.bos_token_id is not None:
            d["bos_token_id"] = self.bos_token_id
        if self.eos_token_ids:
            d["eos_token_id"] = self.eos_token_ids[0] if len(self.eos_token_ids) == 1 else list(self.eos_token_ids)
        return d

    # ------------------------------------------------------------------ the model as data
    def _latent(self, m):
        padded = (m["rot_dim"] + m["kv_rank"] + 15) // 16 * 16
        position = PartSpec("rope", {"head_dim": padded, "rotary_dim": m["rot"]["dims"], "theta": m["rot"]["base"],
                                     "weight_rows": "interleaved"})
        return PartSpec("latent_attention", {
            "n_heads": m["heads"], "head_dim": m["dim"], "rot_dim": m["rot_dim"], "v_dim": m["vdim"], "q_rank": m["q_rank"],
            "kv_rank": m["kv_rank"], "scale": m["scale"], "eps": self.eps, "own_keys": m.get("kv_from") is None,
            "position": position,
            "tensors": {"down_q": "dq", "q_norm": "dq.norm", "q": "uq", "down_kv": "dkv", "kv_norm": "dkv.norm", "up_k": "uk",
                        "up_v": "uv", "out": "o"}}, prefix="mix.")

    def _gla(self, i, m):
        if "decay_rank" not in m:
            raise ConfigError("layer %d: decay_rank is neither in the configuration nor taken from a folder's tensors" % i)
        return PartSpec("gla", {"n_heads": m["heads"], "key_dim": m["dim"], "value_dim": m["vdim"], "decay_rank": m["decay_rank"],
                                "tau": m["tau"], "q_scale": m["dim"] ** -0.5, "eps": self.eps}, prefix="mix.")

    def to_spec(self):
        norm = {"eps": self.eps}
        joining = dict(norm, stream_scale=self.alpha)
        layers, schedule = [], []
        for i, l in enumerate(self.layers):
            m, mlp = l["mixer"], l["mlp"]
            members = {"mixer": self._gla(i, m) if l["type"] == "gla" else self._latent(m),
                       "mixer_norm": PartSpec("layernorm", dict(joining, tensor="norm1"))}
            if mlp is not None:
                r = mlp["router"]
                groups = r.get("groups") or {"count": 1, "keep": 1}
                members["feed_forward"] = PartSpec("moe", {
                    "hidden": mlp["expert"]["ff"], "n_experts": r["experts"], "top": r["top"], "unit": "relu2",
                    "scores": "sigmoid", "groups": groups["count"], "keep_groups": groups["keep"], "weight_scale": r["scale"],
                    "expert_prefix": "e%d.", "tensors": {"correction": "correction"}}, prefix="mlp.")
                members["feed_forward_norm"] = PartSpec("layernorm", dict(joining, tensor="norm2"))
            layers.append(LayerSpec("postnorm_residual", parts=members, prefix="l%d." % i))
            j = m.get("kv_from")
            schedule.append(ScheduleEntry(layer=i, cache=i if j is None else j, writes_cache=j is None))
        pairs = None if self.bigram is None else dict(self.bigram, tensor="bigram")
        return ModelSpec(
            architecture=self.architecture, dim=self.width, vocab_size=self.vocab, max_positions=POSITIONS,
            embedding=PartSpec("token_embedding", {"vocab_size": self.vocab, "tensor": "embed", "scale": self.embedding_scale,
                                                   "pairs": pairs}),
            layers=layers, final_norm=PartSpec("layernorm", dict(norm, tensor="final.norm")),
            head=PartSpec("lm_head", {"vocab_size": self.vocab, "tied": False, "tensor": "head"}),
            schedule=schedule, bos_token_id=self.bos_token_id, eos_token_ids=list(self.eos_token_ids))
