"""Sazavik configuration, read from the design's own ``config.json`` keys.

A decoder whose embedding output goes through a norm before the first layer, whose layers are listed one by one
(``layers``) and whose logits are capped (``logit_softcap``).  A layer normalizes before and after each branch,
x <- x + norm1b(mixer(norm1(x))), x <- x + norm2b(ff(norm2(x))), with RMS norms whose weights are stored around zero.
Mixers (``type``), all grouped-query softmax attention with RMS-normed q and k heads:

``attention``    neighbouring pairs of the first ``rot.dims`` dims turned, chunks of ``mask.size`` positions, a learned sink
                 per head, a gate on the heads' outputs.
``attention_2``  half-split pairs turned, chunks of ``mask.size`` positions.
``attention_3``  biases on its projections, no rotation, queries times a temperature that grows with their position
                 (``q_temp``: coef, every), scores that fall linearly with the distance, a window of ``mask.size`` keys, a
                 gate on the heads' outputs.

With ``kv_from`` a layer has no keys and values of its own: it attends, through its own mask, to those that the named
layer cached.  Feed-forwards (``mlp.kind``, or null for a layer without one): ``dense`` (the clamped gated activation,
``limit``) and ``moe``: ``router.experts`` SiLU-gated experts of which a token uses the ``router.top`` with the largest
sigmoid scores; a score multiplies its expert's input; ``shared``: an expert that every token uses beside them, behind a
sigmoid gate.

Tensors are stored without ``.weight``: ``embed``, ``embed.norm``, ``l<i>.norm1``, ``l<i>.norm1b``, ``l<i>.mix.q``,
``l<i>.mix.q.b``, ``l<i>.mix.q.norm``, ``l<i>.mix.g``, ``l<i>.mix.sink``, ``l<i>.mlp.router``, ``l<i>.mlp.e<k>.up``,
``l<i>.mlp.shared.sg``, ``final.norm``, ``head``.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Tuple

from .mukutar import _integer, _number, _table
from .spec import (SILU_GLU, AttentionSpec, ClampedGLUSpec, ConfigError, InterleavedRopeSpec, LayerSpec, LinearDistanceBiasSpec,
                   MixerSlot, ModelSpec, NoPositionSpec, RmsNormSpec, RopeSpec, RoutedExpertsSpec, ScheduleEntry, SwiGLUSpec,
                   _require)

# a tensor's name in the model -> the name it is stored under
STORED_NAME_RULES = ((r"\.(q|k)_norm\.weight$", r".\1.norm"), (r"_proj\.", "."), (r"\.weight$", ""), (r"\.bias$", ".b"))

FIELD_NAMES = (("attention.head_dim", "layers[].mixer.dim"), ("attention.num_heads", "layers[].mixer.heads"),
               ("routed_experts.num_experts", "layers[].mlp.router.experts"), ("rmsnorm.hidden_size", "width"))

DEFAULT_MAX_CONTEXT = 1 << 20       # the design names no limit: the longest the engine's tables index


@dataclass(frozen=True)
class SazavikLayer:
    type: str
    mixer: AttentionSpec
    mlp: Optional[object]               # the feed-forward's spec, None for a layer without one
    kv_from: Optional[int]              # the layer whose cached keys and values this one reads
    raw: dict                           # the layer's own table, for ``to_dict``


@dataclass(frozen=True)
class SazavikConfig:
    width: int
    vocab: int
    norm_eps: float
    layers: Tuple[SazavikLayer, ...]
    logit_softcap: Optional[float] = None
    max_context: int = DEFAULT_MAX_CONTEXT
    eos_token_id: Optional[int] = None

    architecture_names = ("Sazavik", "sazavik")

    # ------------------------------------------------------------------ reading
    @classmethod
    def from_dict(cls, raw: dict) -> "SazavikConfig":
        width = _integer(raw, "width", "")
        vocab = _integer(raw, "vocab", "")
        eps = _number(_table(raw.get("norm", {}), "norm"), "eps", "norm")
        listed = raw.get("layers")
        if not isinstance(listed, list) or not listed:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        layers = []
        for index, entry in enumerate(listed):
            where = f"layers[{index}]"
            entry = _table(entry, where)
            kind = entry.get("type")
            form = _FORMS.get(kind)
            if form is None:
                raise ConfigError(f"config.json: '{where}.type' is {kind!r}; known: {sorted(_FORMS)}")
            table = _table(entry.get("mixer"), f"{where}.mixer")
            mixer = _attention(table, f"{where}.mixer", eps, form)
            kv_from = None if table.get("kv_from") is None else _integer(table, "kv_from", f"{where}.mixer")
            mlp = None
            if entry.get("mlp") is not None:
                table = _table(entry["mlp"], f"{where}.mlp")
                if table.get("kind") not in _FEED_FORWARDS:
                    raise ConfigError(f"config.json: '{where}.mlp.kind' is {table.get('kind')!r}; "
                                      f"known: {sorted(_FEED_FORWARDS)}")
                mlp = _FEED_FORWARDS[table["kind"]](table, f"{where}.mlp")
            layers.append(SazavikLayer(kind, mixer, mlp, kv_from, entry))
        eos = raw.get("eos_token_id")
        cap = raw.get("logit_softcap")
        config = cls(width=width, vocab=vocab, norm_eps=eps, layers=tuple(layers),
                     logit_softcap=None if cap is None else _number(raw, "logit_softcap", ""),
                     max_context=_integer(raw, "max_context", "", DEFAULT_MAX_CONTEXT),
                     eos_token_id=eos if isinstance(eos, int) and not isinstance(eos, bool) else None)
        config.validate()
        return config

    def to_dict(self) -> dict:
        out = {"architecture": "Sazavik", "layers": [layer.raw for layer in self.layers], "norm": {"eps": self.norm_eps},
               "vocab": self.vocab, "width": self.width}
        if self.logit_softcap is not None:
            out["logit_softcap"] = self.logit_softcap
        if self.max_context != DEFAULT_MAX_CONTEXT:
            out["max_context"] = self.max_context
        return out

    def validate(self) -> None:
        _require(self.width > 0 and self.vocab > 0, "config.json: 'width' and 'vocab' must be positive")
        for index, layer in enumerate(self.layers):
            if layer.kv_from is None:
                continue
            where = f"config.json: 'layers[{index}].mixer.kv_from' names layer {layer.kv_from}"
            _require(0 <= layer.kv_from < index, f"{where}, which does not run before it")
            source = self.layers[layer.kv_from]
            _require(source.kv_from is None, f"{where}, which caches no keys of its own")
            mine, theirs = layer.mixer, source.mixer
            _require((mine.num_kv_heads, mine.head_dim, mine.value_width, _rotation(mine))
                     == (theirs.num_kv_heads, theirs.head_dim, theirs.value_width, _rotation(theirs)),
                     f"{where}, whose kv_heads, dim, vdim or rotation differ")
        self.to_model_spec().validate()

    # ------------------------------------------------------------------ lowering
    def to_model_spec(self) -> ModelSpec:
        norm = RmsNormSpec(eps=self.norm_eps, weight_offset=1.0)
        layers = tuple(
            LayerSpec(prefix=f"l{index}", mixers=(MixerSlot("mix", layer.mixer),), ffn=layer.mlp, mixer_norm=norm,
                      ffn_norm=norm, mixer_norm_name="norm1", ffn_norm_name="norm2", ffn_name="mlp", arrangement="sandwich",
                      mixer_post_norm=norm, ffn_post_norm=norm, mixer_post_norm_name="norm1b",
                      ffn_post_norm_name="norm2b")
            for index, layer in enumerate(self.layers))
        return ModelSpec(
            architecture="Sazavik", hidden_size=self.width, vocab_size=self.vocab, max_context=self.max_context,
            layers=layers,
            schedule=tuple(ScheduleEntry(layer=index, kv_from=layer.kv_from) for index, layer in enumerate(self.layers)),
            final_norm=norm, logit_softcap=self.logit_softcap, embedding_norm=norm, embedding_norm_name="embed.norm",
            embedding_name="embed", final_norm_name="final.norm", lm_head_name="head", root_namespace="",
            stored_name_rules=STORED_NAME_RULES, field_names=FIELD_NAMES)

    # ------------------------------------------------------------------ reports
    def kv_bytes_per_token(self, bytes_per_element: int) -> int:
        """What every layer that caches keeps for one token (windows and chunks bound how many tokens are kept, not this)."""
        return sum(layer.mixer.num_kv_heads * (layer.mixer.head_dim + layer.mixer.value_width) * bytes_per_element
                   for layer in self.layers if layer.kv_from is None)

    def fixed_state_bytes(self, bytes_per_element: int) -> int:
        """No mixer of the design keeps a state."""
        return 0


@dataclass(frozen=True)
class _Form:
    """What tells the design's attentions apart."""
    rotation: Optional[type]        # the position encoding's spec, or None: scores that fall with the distance
    chunked: bool                   # ``mask.size`` is a chunk's, not a window's
    sink: bool = False
    gate: bool = False
    bias: bool = False


_FORMS = {"attention": _Form(InterleavedRopeSpec, chunked=True, sink=True, gate=True),
          "attention_2": _Form(RopeSpec, chunked=True),
          "attention_3": _Form(None, chunked=False, gate=True, bias=True)}


def _rotation(spec: AttentionSpec):
    """What a layer's cached keys have gone through by position: the rotation, or nothing."""
    return spec.position if isinstance(spec.position, (RopeSpec, InterleavedRopeSpec)) else None


def _attention(mixer: dict, where: str, eps: float, form: _Form) -> AttentionSpec:
    heads = _integer(mixer, "heads", where)
    dim = _integer(mixer, "dim", where)
    temperature = None
    if form.rotation is None:
        position = LinearDistanceBiasSpec(num_heads=heads)
        if mixer.get("q_temp") is not None:
            table = _table(mixer["q_temp"], f"{where}.q_temp")
            every = _number(table, "every", f"{where}.q_temp")
            _require(every == int(every) and every > 0, f"config.json: '{where}.q_temp.every' must be a positive whole number")
            temperature = (_number(table, "coef", f"{where}.q_temp"), int(every))
    elif mixer.get("rot") is not None:
        rot = _table(mixer["rot"], f"{where}.rot")
        position = form.rotation(theta=_number(rot, "base", f"{where}.rot"), rotary_dim=_integer(rot, "dims", f"{where}.rot", dim))
    else:
        position = NoPositionSpec()
    size = None
    if mixer.get("mask") is not None:
        mask = _table(mixer["mask"], f"{where}.mask")
        size = None if mask.get("size") is None else _integer(mask, "size", f"{where}.mask")
    return AttentionSpec(num_heads=heads, num_kv_heads=_integer(mixer, "kv_heads", where, heads), head_dim=dim,
                         scale=_number(mixer, "scale", where), position=position, window=None if form.chunked else size,
                         chunk=size if form.chunked else None, qkv_bias=form.bias, out_bias=form.bias,
                         value_dim=_integer(mixer, "vdim", where, dim), sink=form.sink, head_norm="before_rotation",
                         head_norm_weight=True, head_norm_eps=eps, out_gate=form.gate, query_temperature=temperature,
                         own_rows=mixer.get("kv_from") is None)


def _dense(mlp: dict, where: str) -> SwiGLUSpec:
    return SwiGLUSpec(intermediate_size=_integer(mlp, "ff", where), activation="clamped",
                      clamp=ClampedGLUSpec(limit=_number(mlp, "limit", where)))


def _moe(mlp: dict, where: str) -> RoutedExpertsSpec:
    expert = _table(mlp.get("expert"), f"{where}.expert")
    router = _table(mlp.get("router"), f"{where}.router")
    shared_size = None
    if mlp.get("shared") is not None:
        shared_size = _integer(_table(mlp["shared"], f"{where}.shared"), "ff", f"{where}.shared")
    return RoutedExpertsSpec(num_experts=_integer(router, "experts", f"{where}.router"),
                             top_k=_integer(router, "top", f"{where}.router"),
                             expert_size=_integer(expert, "ff", f"{where}.expert"), activation=SILU_GLU,
                             shared_size=shared_size, shared_activation=None if shared_size is None else SILU_GLU,
                             routing="sigmoid_then_top", renormalize=False, corrected=False, input_weighted=True)


_FEED_FORWARDS = {"dense": _dense, "moe": _moe}
