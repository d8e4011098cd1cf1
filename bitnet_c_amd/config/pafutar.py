"""Pafutar: a decoder whose config.json lists its layers one by one.  The norms stand behind the sums, and a layer's
halves read the residual stream itself (parts/block.py, "postnorm"):

    x <- norm1(alpha x + ls1 mixer(h));   x <- norm2(alpha x + ls2 ff(x))      plain RMSNorms with weights [width]

with h = x + (x' - x) * shift, x' the previous token's x (parts/shift.py), and ls1, ls2, shift vectors [width].  The
embedding's rows are multiplied by a constant and a learned vector per position is added.

The mixer is "attention" (parts/attention.py): grouped-query attention without a rotation whose values are the key
projections themselves; biases on the query and key projections; an RMSNorm without weights over every query and key head;
scores times a number per head, less slope_h times the distance, slope_h = 2^(-8 (h + 1) / heads); a sliding window beside
which a sequence's first tokens stay visible; the heads' outputs times sigmoid(W_g h).  The feed-forward is "dense" (squared
relu, no gate); "mlp": null leaves the second half out.  "weights_of": j runs layer j's block once more, norms and vectors
included, over other pages and another state row: the plan's schedule names that block twice.

config.json keys: architecture, vocab, width, max_positions, norm.eps, embedding.scale, postln_alpha,
  layers[] = {type: "attention", mixer, mlp, weights_of?} with
  mixer   {heads, kv_heads, dim, vdim, scale, mask: {size, keep_first}}
  mlp     {kind: "dense", ff} | null

Tensor names of the folder (linear weights [out, in]): embed, pos, head, final.norm, and for layer i under l<i>.:
  norm1, norm2, ls1, ls2, shift, mix.{q,k,g,o}, mix.q.b, mix.k.b, mix.temp, mlp.{up,down}
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Tuple

from ..engine.plan import LayerPlan, ModelPlan, ScheduleEntry
from ..parts.base import PartSpec
from .base import Architecture, ConfigError, _positive_int, register_architecture

NAME = "Pafutar"
SLOPE_RANGE = 8.0             # the distance slopes run from 2^(-8 / heads) down to 2^-8; the design fixes it


def distance_slopes(heads: int) -> Tuple[float, ...]:
    return tuple(2.0 ** (-SLOPE_RANGE * (h + 1) / heads) for h in range(heads))


def _number(raw: dict, key: str, what: str, positive: bool = True) -> float:
    v = raw.get(key)
    if isinstance(v, bool) or not isinstance(v, (int, float)) or (positive and not v > 0):
        raise ConfigError(f"config.json: {what}.{key} must be a {'positive ' if positive else ''}number, got {v!r}")
    return float(v)


def _object(raw, what: str) -> dict:
    if not isinstance(raw, dict):
        raise ConfigError(f"config.json: {what} must be an object, got {raw!r}")
    return raw


@dataclass(frozen=True)
class WindowAttentionSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int = 0             # 0: no mask but the causal one
    keep_first: int = 0

    def to_dict(self):
        d = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.window:
            d["mask"] = {"size": self.window, "keep_first": self.keep_first}
        return d


@dataclass(frozen=True)
class PafutarLayer:
    type: str                                  # "attention"
    mixer: WindowAttentionSizes
    ff: Optional[int]                          # the dense feed-forward's inner width; None: the layer has none
    weights_of: Optional[int] = None

    def to_dict(self):
        d = {"type": self.type, "mixer": self.mixer.to_dict(),
             "mlp": None if self.ff is None else {"kind": "dense", "ff": self.ff}}
        if self.weights_of is not None:
            d["weights_of"] = self.weights_of
        return d


@dataclass(frozen=True)
class PafutarConfig:
    vocab: int
    width: int
    max_positions: int
    eps: float
    embedding_scale: float
    alpha: float
    layers: Tuple[PafutarLayer, ...]

    MIXER_TYPES = ("attention",)

    @staticmethod
    def _mixer(raw, where: str) -> WindowAttentionSizes:
        m = _object(raw, where + ".mixer")
        heads, dim = _positive_int(m, "heads"), _positive_int(m, "dim")
        kv_heads, vdim = _positive_int(m, "kv_heads", heads), _positive_int(m, "vdim", dim)
        if heads % kv_heads:
            raise ConfigError(f"config.json: {where}: {heads} heads are not a multiple of {kv_heads} kv_heads")
        if vdim != dim:
            raise ConfigError(f"config.json: {where}.mixer: the values are the keys, so vdim {vdim} must equal dim {dim}")
        window = keep = 0
        if m.get("mask") is not None:
            mask = _object(m["mask"], where + ".mixer.mask")
            window, keep = _positive_int(mask, "size"), mask.get("keep_first", 0)
            if isinstance(keep, bool) or not isinstance(keep, int) or keep < 0:
                raise ConfigError(f"config.json: {where}.mixer.mask.keep_first must be a number of tokens, got {keep!r}")
        return WindowAttentionSizes(heads, kv_heads, dim, vdim, _number(m, "scale", where + ".mixer"), window, keep)

    @classmethod
    def from_dict(cls, raw: dict) -> "PafutarConfig":
        norm, emb = _object(raw.get("norm"), "norm"), _object(raw.get("embedding", {}), "embedding")
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
            mlp, ff = L.get("mlp"), None
            if mlp is not None:
                mlp = _object(mlp, where + ".mlp")
                if mlp.get("kind") != "dense":
                    raise ConfigError(f"config.json: {where}.mlp.kind {mlp.get('kind')!r} is not supported (supported: 'dense')")
                ff = _positive_int(mlp, "ff")
            wo = L.get("weights_of")
            if wo is not None and (isinstance(wo, bool) or not isinstance(wo, int) or not 0 <= wo < len(layers_raw) or wo == i):
                raise ConfigError(f"config.json: {where}.weights_of {wo!r} names no other layer")
            layers.append(PafutarLayer(kind, cls._mixer(L.get("mixer"), where), ff, wo))
        for i, L in enumerate(layers):
            if L.weights_of is not None:
                src = layers[L.weights_of]
                if src.weights_of is not None:
                    raise ConfigError(f"config.json: layers[{i}] uses the weights of layers[{L.weights_of}], which has none of its own")
                if (src.type, src.mixer, src.ff) != (L.type, L.mixer, L.ff):
                    raise ConfigError(f"config.json: layers[{i}] uses the weights of layers[{L.weights_of}] but differs from it")
        return cls(vocab=_positive_int(raw, "vocab"), width=_positive_int(raw, "width"),
                   max_positions=_positive_int(raw, "max_positions"), eps=_number(norm, "eps", "norm"),
                   embedding_scale=_number(emb, "scale", "embedding") if "scale" in emb else 1.0,
                   alpha=_number(raw, "postln_alpha", "config"), layers=tuple(layers))

    def to_dict(self) -> dict:
        return {"architecture": NAME, "vocab": self.vocab, "width": self.width, "max_positions": self.max_positions,
                "norm": {"eps": self.eps}, "embedding": {"scale": self.embedding_scale}, "postln_alpha": self.alpha,
                "layers": [L.to_dict() for L in self.layers]}


def _mixer_spec(c: PafutarConfig, m: WindowAttentionSizes):
    """(mixer spec, the mixer's local tensor names -> names under l<i>.mix.)"""
    spec = PartSpec.of("attention", hidden=c.width, n_heads=m.heads, n_kv_heads=m.kv_heads, head_dim=m.dim, scale=m.scale,
                       position=PartSpec.of("none"), window=m.window, keep_first=m.keep_first if m.window else 0, bias="qk",
                       qk_norm_eps=c.eps, qk_norm_weight=False, head_temp=True, distance_slopes=distance_slopes(m.heads),
                       value_is_key=True, out_gate=True)
    return spec, {"wq": "q", "wk": "k", "wg": "g", "wo": "o", "bq": "q.b", "bk": "k.b", "temp": "temp"}


def build_pafutar_plan(c: PafutarConfig) -> ModelPlan:
    norm = PartSpec.of("rmsnorm", dim=c.width, eps=c.eps)
    layers, index = [], {}                  # index: config layer -> its place among the layers that own tensors
    for i, L in enumerate(c.layers):
        if L.weights_of is not None:
            continue
        p = f"l{i}."
        mixer, mixer_names = _mixer_spec(c, L.mixer)
        ffn = PartSpec.of("dense", hidden=c.width, intermediate=L.ff, activation="relu2") if L.ff is not None else None
        names = {"mixer_norm.weight": p + "norm1", "mixer_gain": p + "ls1", "shift.mu": p + "shift"}
        names.update({"mixer." + local: p + "mix." + name for local, name in mixer_names.items()})
        if ffn is not None:
            names.update({"ffn_norm.weight": p + "norm2", "ffn_gain": p + "ls2", "ffn.w_up": p + "mlp.up", "ffn.w_down": p + "mlp.down"})
        block = PartSpec.of("postnorm", hidden=c.width, mixer=mixer, ffn=ffn, mixer_norm=norm,
                            ffn_norm=norm if ffn is not None else None, alpha=c.alpha, layer_scale=True, token_shift=True)
        index[i] = len(layers)
        layers.append(LayerPlan(block=block, names=names))
    schedule = [ScheduleEntry(index[L.weights_of if L.weights_of is not None else i]) for i, L in enumerate(c.layers)]
    plan = ModelPlan(vocab_size=c.vocab, hidden_size=c.width, layers=layers, schedule=schedule, final_norm=norm,
                     embedding_name="embed", final_norm_names={"weight": "final.norm"}, lm_head_name="head",
                     max_positions=c.max_positions, position_table_name="pos", embedding_multiplier=c.embedding_scale)
    plan.validate()
    return plan


PAFUTAR = register_architecture(Architecture(name=NAME, config_cls=PafutarConfig, build_plan=build_pafutar_plan,
                                             aliases=("pafutar",)))
