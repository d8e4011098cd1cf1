"""Zenasun: a decoder whose config.json lists its layers one by one.  A layer's mixer and feed-forward read the same
residual stream, each under a norm of its own, and join it together (parts/block.py, "parallel_prenorm"):

    x += mixer(norm1(x)) + ff(norm2(x))            RMSNorms whose stored weight w means 1 + w, as the model's last norm

Two kinds of mixers:

  "latent_attention"  causal attention whose queries pass a normed latent and whose keys and values are projections of one
                      normed latent per token, beside one rotated key part that all heads share (neighbouring pairs), with
                      a learned sink per head in the softmax (parts/latent.py)
  "retention"         linear attention with a matrix state per head and a decay that is a constant of the head, over
                      rotated queries and keys (split-half pairs); every head's output is normed by itself and gated by a
                      silu (parts/recurrent.py)

and one kind of feed-forward, "moe": gated experts and identity experts (whose output is their input), chosen by softmax
score + a correction inside the best groups of neighbours, weighted by the plain scores of the chosen over their sum
(parts/moe.py); "mlp": null leaves it out.  A layer with "weights_of": j has no tensors of its own: it runs layer j's
weights with a cache or state of its own, which the plan's schedule says by naming layer j twice.  The embedding's rows
are multiplied by a constant on their way in; the embedding itself is the output matrix, whose logits pass a soft-cap.

config.json keys: architecture, vocab, width, norm.eps, embedding.scale, logit_softcap, layers[] = {type, mixer, mlp,
weights_of?} with
  latent mixer      {heads, dim, rot_dim, vdim, kv_rank, q_rank, scale, rot: {base, dims}}
  retention mixer   {heads, dim, vdim, decay: [one per head], rot: {base, dims}}
  mlp               {kind: "moe", expert: {ff}, router: {experts, top, identity, groups: {count, keep}}} | null

Tensor names of the folder (linear weights [out, in]): embed, final.norm, and for layer i under l<i>.:
  norm1, norm2
  latent:     mix.dq, mix.dq.norm, mix.uq, mix.dkv, mix.dkv.norm, mix.uk, mix.uv, mix.sink, mix.o
  retention:  mix.{q,k,v,g,o}
  moe:        mlp.router, mlp.correction, mlp.e<n>.{gate,up,down}
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Tuple, Union

from ..engine.plan import LayerPlan, ModelPlan, ScheduleEntry
from ..parts.base import PartSpec
from .base import Architecture, ConfigError, _positive_int, register_architecture
from .fazopel import WEIGHT_FLOOR, _number, _object
from .mutirax import LatentSizes, Rotation, _rotation

NAME = "Zenasun"

NORM_OFFSET = 1.0             # a stored norm weight w means NORM_OFFSET + w (the same in every model of the design)


def _count(raw: dict, key: str, where: str, default: int = 0) -> int:
    """A whole number of 0 or more; null and a missing key are the default."""
    v = raw.get(key)
    if v is None:
        return default
    if isinstance(v, bool) or not isinstance(v, int) or v < 0:
        raise ConfigError(f"config.json: {where}.{key} must be a whole number of 0 or more, got {v!r}")
    return v


@dataclass(frozen=True)
class RetentionSizes:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]
    rot: Optional[Rotation]

    def to_dict(self):
        d = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "decay": list(self.decay)}
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        return d


@dataclass(frozen=True)
class GroupedMoeSizes:
    experts: int
    identity: int
    top: int
    groups: Tuple[int, int]                    # (count, keep); (1, 1): no groups
    ff: int

    def to_dict(self):
        return {"kind": "moe", "expert": {"ff": self.ff},
                "router": {"experts": self.experts, "identity": self.identity, "top": self.top,
                           "groups": {"count": self.groups[0], "keep": self.groups[1]}}}


@dataclass(frozen=True)
class ZenasunLayer:
    type: str                                  # "latent_attention" | "retention"
    mixer: Union[LatentSizes, RetentionSizes]
    mlp: Optional[GroupedMoeSizes]
    weights_of: Optional[int] = None

    def to_dict(self):
        d = {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}
        if self.weights_of is not None:
            d["weights_of"] = self.weights_of
        return d


@dataclass(frozen=True)
class ZenasunConfig:
    vocab: int
    width: int
    eps: float
    embedding_scale: float
    logit_softcap: float                       # 0: none
    layers: Tuple[ZenasunLayer, ...]

    MIXER_TYPES = ("latent_attention", "retention")
    MLP_KINDS = ("moe",)

    @staticmethod
    def _mixer(kind: str, raw, where: str):
        w = where + ".mixer"
        m = _object(raw, w)
        heads, dim = _positive_int(m, "heads"), _positive_int(m, "dim")
        vdim = _positive_int(m, "vdim", dim)
        if kind == "retention":
            decay = m.get("decay")
            if (not isinstance(decay, list) or len(decay) != heads
                    or any(isinstance(d, bool) or not isinstance(d, (int, float)) or not 0.0 <= d <= 1.0 for d in decay)):
                raise ConfigError(f"config.json: {w}.decay must list one number in [0, 1] for each of the {heads} heads")
            return RetentionSizes(heads, dim, vdim, tuple(float(d) for d in decay), _rotation(m.get("rot"), w + ".rot", dim))
        rot_dim = _count(m, "rot_dim", w)
        if rot_dim % 2:
            raise ConfigError(f"config.json: {w}.rot_dim must be even, got {rot_dim}")
        rot = _rotation(m.get("rot"), w + ".rot", rot_dim) if rot_dim else None
        if rot_dim and (rot is None or rot.dims != rot_dim):
            raise ConfigError(f"config.json: {w}: a rotated part of {rot_dim} dimensions needs rot with as many, got {m.get('rot')!r}")
        return LatentSizes(heads, dim, rot_dim, vdim, _positive_int(m, "kv_rank"), _positive_int(m, "q_rank"),
                           _number(m, "scale", w), rot)

    @classmethod
    def _mlp(cls, raw, where: str):
        if raw is None:
            return None
        w = where + ".mlp"
        m = _object(raw, w)
        if m.get("kind") not in cls.MLP_KINDS:
            raise ConfigError(f"config.json: {w}.kind {m.get('kind')!r} is not one of {cls.MLP_KINDS}")
        router = _object(m.get("router"), w + ".router")
        experts, top, identity = _positive_int(router, "experts"), _positive_int(router, "top"), _count(router, "identity", w + ".router")
        groups = (1, 1)
        if router.get("groups") is not None:
            g = _object(router["groups"], w + ".router.groups")
            groups = (_positive_int(g, "count"), _positive_int(g, "keep"))
        n = experts + identity
        if n % groups[0] or groups[1] > groups[0] or top > groups[1] * (n // groups[0]):
            raise ConfigError(f"config.json: {w}.router: the best {groups[1]} of {groups[0]} equal groups of {n} experts do not "
                              f"hold the top {top}")
        return GroupedMoeSizes(experts, identity, top, groups, _positive_int(_object(m.get("expert"), w + ".expert"), "ff"))

    @classmethod
    def from_dict(cls, raw: dict) -> "ZenasunConfig":
        norm = _object(raw.get("norm"), "norm")
        layers_raw = raw.get("layers")
        if not isinstance(layers_raw, list) or not layers_raw:
            raise ConfigError("config.json: layers must be a list with at least one entry")
        layers = []
        for i, L in enumerate(layers_raw):
            where = f"layers[{i}]"
            L = _object(L, where)
            kind = L.get("type")
            if kind not in cls.MIXER_TYPES:
                raise ConfigError(f"config.json: {where}.type {kind!r} is not one of {cls.MIXER_TYPES}")
            wo = L.get("weights_of")
            if wo is not None and (isinstance(wo, bool) or not isinstance(wo, int) or not 0 <= wo < len(layers_raw) or wo == i):
                raise ConfigError(f"config.json: {where}.weights_of {wo!r} names no other layer")
            layers.append(ZenasunLayer(kind, cls._mixer(kind, L.get("mixer"), where), cls._mlp(L.get("mlp"), where), wo))
        for i, L in enumerate(layers):
            if L.weights_of is not None:
                src = layers[L.weights_of]
                if src.weights_of is not None:
                    raise ConfigError(f"config.json: layers[{i}] uses the weights of layers[{L.weights_of}], which has none of its own")
                if (src.type, src.mixer, src.mlp) != (L.type, L.mixer, L.mlp):
                    raise ConfigError(f"config.json: layers[{i}] uses the weights of layers[{L.weights_of}] but differs from it")
        emb = _object(raw.get("embedding") or {}, "embedding")
        return cls(vocab=_positive_int(raw, "vocab"), width=_positive_int(raw, "width"), eps=_number(norm, "eps", "norm"),
                   embedding_scale=_number(emb, "scale", "embedding") if "scale" in emb else 1.0,
                   logit_softcap=_number(raw, "logit_softcap", "config") if raw.get("logit_softcap") is not None else 0.0,
                   layers=tuple(layers))

    def to_dict(self) -> dict:
        d = {"architecture": NAME, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
             "embedding": {"scale": self.embedding_scale}, "layers": [L.to_dict() for L in self.layers]}
        if self.logit_softcap:
            d["logit_softcap"] = self.logit_softcap
        return d


def _mixer_spec(c: ZenasunConfig, L: ZenasunLayer):
    """(mixer spec, the mixer's local tensor names -> names under l<i>.mix.)"""
    m = L.mixer
    if L.type == "retention":
        rot = dict(rope_dims=m.rot.dims, rope_theta=m.rot.base) if m.rot is not None else {}
        spec = PartSpec.of("retention", hidden=c.width, n_heads=m.heads, head_dim=m.dim, v_head_dim=m.vdim, decay=m.decay, eps=c.eps,
                           **rot)
        return spec, {"wq": "q", "wk": "k", "wv": "v", "wg": "g", "wo": "o"}
    spec = PartSpec.of("latent_attention", hidden=c.width, n_heads=m.heads, head_dim=m.dim, v_head_dim=m.vdim, kv_rank=m.kv_rank,
                       scale=m.scale, eps=c.eps, gate=False, q_rank=m.q_rank, rot_dim=m.rot_dim,
                       rot_theta=m.rot.base if m.rot is not None else 10000.0, rot_interleaved=True, sink=True)
    return spec, {"wdq": "dq", "dq_norm": "dq.norm", "wuq": "uq", "wdkv": "dkv", "dkv_norm": "dkv.norm", "wuk": "uk", "wuv": "uv",
                  "sink": "sink", "wo": "o"}


def _ffn_spec(c: ZenasunConfig, mlp: GroupedMoeSizes, prefix: str):
    """(feed-forward spec, its local tensor names -> names of the folder)"""
    spec = PartSpec.of("moe", hidden=c.width, n_experts=mlp.experts, identity_experts=mlp.identity, groups=mlp.groups, top_k=mlp.top,
                       intermediate=mlp.ff, activation="silu", gated=True, scoring="softmax", renormalize=True, weight_on="output",
                       choice_bias=True, weight_floor=WEIGHT_FLOOR)
    names = {"router": prefix + "router", "correction": prefix + "correction"}
    for e in range(mlp.experts):
        names.update({f"e{e}.w_gate": f"{prefix}e{e}.gate", f"e{e}.w_up": f"{prefix}e{e}.up", f"e{e}.w_down": f"{prefix}e{e}.down"})
    return spec, names


def build_zenasun_plan(c: ZenasunConfig) -> ModelPlan:
    norm = PartSpec.of("rmsnorm", dim=c.width, eps=c.eps, offset=NORM_OFFSET)
    layers, index = [], {}                  # index: config layer -> its place among the layers that own tensors
    for i, L in enumerate(c.layers):
        if L.weights_of is not None:
            continue
        p = f"l{i}."
        mixer, mixer_names = _mixer_spec(c, L)
        names = {"mixer_norm.weight": p + "norm1"}
        names.update({"mixer." + local: p + "mix." + name for local, name in mixer_names.items()})
        ffn = None
        if L.mlp is not None:
            ffn, ffn_names = _ffn_spec(c, L.mlp, p + "mlp.")
            names["ffn_norm.weight"] = p + "norm2"
            names.update({"ffn." + local: name for local, name in ffn_names.items()})
        block = PartSpec.of("parallel_prenorm", mixer=mixer, ffn=ffn, mixer_norm=norm, ffn_norm=norm if ffn is not None else None)
        index[i] = len(layers)
        layers.append(LayerPlan(block=block, names=names))
    schedule = [ScheduleEntry(index[L.weights_of if L.weights_of is not None else i]) for i, L in enumerate(c.layers)]
    plan = ModelPlan(vocab_size=c.vocab, hidden_size=c.width, layers=layers, schedule=schedule, final_norm=norm,
                     embedding_name="embed", final_norm_names={"weight": "final.norm"}, lm_head_name=None,
                     embedding_multiplier=c.embedding_scale, logit_softcap=c.logit_softcap)
    plan.validate()
    return plan


ZENASUN = register_architecture(Architecture(name=NAME, config_cls=ZenasunConfig, build_plan=build_zenasun_plan,
                                             aliases=("zenasun",)))
