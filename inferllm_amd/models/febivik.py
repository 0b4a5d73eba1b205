"""Febivik: a decoder whose sublayers read the residual stream itself and pass a layer norm behind
(x <- x + norm(sublayer(x))), with three kinds of mixer in any order: softmax attention with biases,
a norm a q and k head, a partial rotation with linear scaling and a sliding window beside which the
sequence's first tokens stay visible; lightning attention with one fixed decay a head; and a
generalized delta rule with a decay, a removal rate and a unit key per head and channel.
Feed-forwards are dense with the xIELU activation, or a mixture of squared-ReLU experts with a
softmax router and a shared expert.  The head is a matrix of its own.

This file holds what is specific to the design: the keys of its config.json, their checks, the
tensor names of its checkpoints and the translation into a `ModelSpec` of generic parts.

    config.json
      architecture: "Febivik"; vocab; width; norm.eps; max_positions?
      layers: [{type: "attention", mixer: {heads, kv_heads, dim, vdim, scale, mask: {size, keep_first?}?,
                                           rot: {base, dims, scaling: {factor}?}?}, mlp}
             | {type: "lightning", mixer: {heads, dim, vdim, decay: [a number a head]}, mlp}
             | {type: "general_delta", mixer: {heads, dim, rank?}, mlp}]
      mlp: null | {kind: "dense", ff} | {kind: "moe", expert: {ff}, router: {experts, top, scale?}, shared: {ff}?}
    tensors
      embed; head; final.norm, final.norm.b; l<i>.norm1, .norm1.b and, with a feed-forward, .norm2, .norm2.b
      attention (l<i>.mix.): q, q.b, k, k.b, v, v.b, q.norm [dim], k.norm [dim], o
      lightning: q, k, v, g, norm [heads vdim], o
      general_delta: r, k, v, g, a, a.b, w1 [rank, width], w2 [heads dim, rank], w0, norm [heads dim], o
      l<i>.mlp.{up, down, act [2]} | l<i>.mlp.{router, e<j>.{up, down}, shared.{up, down}}

The rank of the decays' low-rank map is the first size of `w1`; a configuration may state it as
`mixer.rank` (random weights need it).  Positions have no limit of their own in the configuration;
`max_positions` (optional key) sizes the angle tables and defaults to 65,536.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import List, Optional

from ..config.registry import ConfigError, register_architecture
from ..config.spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry

DEFAULT_MAX_POSITIONS = 65536
DEFAULT_DECAY_RANK = 16


def _get(d: dict, key: str, where: str, kind=None):
    if not isinstance(d, dict) or key not in d:
        raise ConfigError(f"config.json of Febivik lacks {where}{key}")
    v = d[key]
    if kind == "int":
        if not isinstance(v, int) or isinstance(v, bool) or v <= 0:
            raise ConfigError(f"{where}{key} must be a positive integer, got {v!r}")
    elif kind == "float":
        if isinstance(v, bool) or not isinstance(v, (int, float)) or not float(v) > 0:
            raise ConfigError(f"{where}{key} must be a positive number, got {v!r}")
    return v


def _check_attention(m: dict, at: str) -> None:
    for k in ("heads", "kv_heads", "dim", "vdim"):
        _get(m, k, at, "int")
    if m["heads"] % m["kv_heads"]:
        raise ConfigError(f"{at}heads {m['heads']} must be a multiple of kv_heads {m['kv_heads']}")
    _get(m, "scale", at, "float")
    if m.get("mask"):
        _get(m["mask"], "size", at + "mask.", "int")
        keep = m["mask"].get("keep_first", 0)
        if not isinstance(keep, int) or isinstance(keep, bool) or keep < 0:
            raise ConfigError(f"{at}mask.keep_first must be a non-negative integer, got {keep!r}")
    if m.get("rot"):
        rot = m["rot"]
        _get(rot, "base", at + "rot.", "float")
        dims = _get(rot, "dims", at + "rot.", "int")
        if dims % 2 or dims > m["dim"]:
            raise ConfigError(f"{at}rot.dims {dims} must be even and at most dim {m['dim']}")
        if rot.get("scaling"):
            _get(rot["scaling"], "factor", at + "rot.scaling.", "float")


def _check_lightning(m: dict, at: str) -> None:
    for k in ("heads", "dim", "vdim"):
        _get(m, k, at, "int")
    decay = _get(m, "decay", at)
    ok = isinstance(decay, list) and len(decay) == m["heads"] and all(
        isinstance(g, (int, float)) and not isinstance(g, bool) and 0.0 <= float(g) <= 1.0 for g in decay)
    if not ok:
        raise ConfigError(f"{at}decay must list one number in [0, 1] for each of {m['heads']} heads, got {decay!r}")


def _check_general_delta(m: dict, at: str) -> None:
    for k in ("heads", "dim") + (("rank",) if "rank" in m else ()):
        _get(m, k, at, "int")


_MIXERS = {"attention": _check_attention, "lightning": _check_lightning, "general_delta": _check_general_delta}


def _check_mlp(mlp: dict, at: str) -> None:
    kind = _get(mlp, "kind", at)
    if kind == "dense":
        _get(mlp, "ff", at, "int")
    elif kind == "moe":
        r = _get(mlp, "router", at)
        n, top = _get(r, "experts", at + "router.", "int"), _get(r, "top", at + "router.", "int")
        if top > n:
            raise ConfigError(f"{at}router: {top} of {n} experts cannot be chosen")
        if "scale" in r:
            _get(r, "scale", at + "router.", "float")
        _get(_get(mlp, "expert", at), "ff", at + "expert.", "int")
        if mlp.get("shared"):
            _get(mlp["shared"], "ff", at + "shared.", "int")
    else:
        raise ConfigError(f"{at}kind {kind!r} is not a feed-forward of this design (dense, moe)")


@register_architecture("Febivik")
@dataclass
class FebivikConfig:
    vocab: int
    width: int
    eps: float
    layers: List[dict] = field(default_factory=list)
    max_positions: int = DEFAULT_MAX_POSITIONS

    architecture = "Febivik"
    cli_type_names = ("febivik",)

    # ------------------------------------------------------------ reading
    @classmethod
    def from_dict(cls, d: dict) -> "FebivikConfig":
        layers = _get(d, "layers", "")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("layers must be a list with at least one layer")
        cfg = cls(vocab=_get(d, "vocab", "", "int"), width=_get(d, "width", "", "int"),
                  eps=float(_get(_get(d, "norm", ""), "eps", "norm.", "float")),
                  layers=copy.deepcopy(layers),
                  max_positions=int(d.get("max_positions", DEFAULT_MAX_POSITIONS)))
        cfg.validate()
        return cfg

    def validate(self) -> None:
        if self.max_positions <= 0:
            raise ConfigError("max_positions must be positive")
        for i, layer in enumerate(self.layers):
            at = f"layers[{i}]."
            kind = _get(layer, "type", at)
            if kind not in _MIXERS:
                raise ConfigError(f"{at}type {kind!r} is not a mixer of this design ({', '.join(_MIXERS)})")
            _MIXERS[kind](_get(layer, "mixer", at), at + "mixer.")
            if layer.get("mlp") is not None:
                _check_mlp(layer["mlp"], at + "mlp.")

    def to_dict(self) -> dict:
        d = {"architecture": self.architecture, "layers": copy.deepcopy(self.layers), "norm": {"eps": self.eps},
             "vocab": self.vocab, "width": self.width}
        if self.max_positions != DEFAULT_MAX_POSITIONS:
            d["max_positions"] = self.max_positions
        return d

    def with_tensor_shapes(self, shapes: dict) -> "FebivikConfig":
        """The configuration with the sizes that only a folder's tensors state (`shapes`: tensor name
        -> shape): the rank of a general_delta layer's decay map."""
        cfg = copy.deepcopy(self)
        for i, layer in enumerate(cfg.layers):
            if layer["type"] == "general_delta" and f"l{i}.mix.w1" in shapes:
                layer["mixer"]["rank"] = int(shapes[f"l{i}.mix.w1"][0])
        return cfg

    # ------------------------------------------------------------ translation
    def _mixer(self, p: str, kind: str, m: dict):
        """(mixer, position encoding of the layer or None)."""
        E = self.width
        names = lambda *ns: {n: p + n for n in ns}
        if kind == "lightning":
            return PartSpec("lightning_attention",
                            {"hidden_size": E, "num_heads": m["heads"], "key_dim": m["dim"], "value_dim": m["vdim"],
                             "decay": [float(g) for g in m["decay"]], "eps": self.eps},
                            names("q", "k", "v", "g", "o", "norm")), None
        if kind == "general_delta":
            return PartSpec("removal_delta_rule",
                            {"hidden_size": E, "num_heads": m["heads"], "dim": m["dim"],
                             "decay_rank": int(m.get("rank", DEFAULT_DECAY_RANK)), "eps": self.eps},
                            {**names("r", "k", "v", "g", "a", "w1", "w2", "w0", "norm", "o"), "a_bias": p + "a.b"}), None
        mask, rot = m.get("mask") or {}, m.get("rot") or None
        position = None if rot is None else PartSpec(
            "rotary", {"head_dim": m["dim"], "rotary_dim": int(rot["dims"]), "theta": float(rot["base"]),
                       "pairing": "half", "max_positions": self.max_positions,
                       "scaling": {"factor": float(rot["scaling"]["factor"])} if rot.get("scaling") else None})
        return PartSpec(
            "gated_attention",
            {"hidden_size": E, "num_heads": m["heads"], "num_kv_heads": m["kv_heads"], "key_dim": m["dim"],
             "value_dim": m["vdim"], "softmax_scale": float(m["scale"]), "window": mask.get("size"),
             "keep_first": int(mask.get("keep_first", 0)) if mask else 0, "qk_norm": "head_weighted",
             "eps": self.eps, "bias": True},
            {**names("q", "k", "v", "o"), "q_norm": p + "q.norm", "k_norm": p + "k.norm", "q_bias": p + "q.b",
             "k_bias": p + "k.b", "v_bias": p + "v.b"}), position

    def _feed_forward(self, p: str, mlp: Optional[dict]) -> PartSpec:
        if mlp is None:
            return PartSpec("none")
        if mlp["kind"] == "dense":
            return PartSpec("dense_activation", {"hidden_size": self.width, "intermediate_size": int(mlp["ff"]),
                                                 "activation": "xielu"},
                            {k: p + k for k in ("up", "down", "act")})
        r, shared = mlp["router"], mlp.get("shared") or None
        parts = [f"e{j}" for j in range(int(r["experts"]))] + (["shared"] if shared else [])
        return PartSpec("routed_experts",
                        {"hidden_size": self.width, "expert_size": int(mlp["expert"]["ff"]),
                         "num_experts": int(r["experts"]), "top": int(r["top"]), "correction": False,
                         "shared_size": int(shared["ff"]) if shared else 0, "shared_gate": False,
                         "activation": "relu_squared", "router_scale": float(r.get("scale", 1.0))},
                        {"router": p + "router", **{f"{e}.{t}": f"{p}{e}.{t}" for e in parts for t in ("up", "down")}})

    def to_spec(self) -> ModelSpec:
        E, V = self.width, self.vocab
        norm = lambda name: PartSpec("layer_norm", {"size": E, "eps": self.eps}, {"weight": name, "bias": name + ".b"})
        layers = []
        for i, layer in enumerate(self.layers):
            mlp = layer.get("mlp")
            mixer, position = self._mixer(f"l{i}.mix.", layer["type"], layer["mixer"])
            layers.append(LayerSpec(
                block="post_norm", mixer=mixer, feed_forward=self._feed_forward(f"l{i}.mlp.", mlp),
                mixer_norm=norm(f"l{i}.norm1"),
                feed_forward_norm=norm(f"l{i}.norm2") if mlp is not None else None, position=position))
        return ModelSpec(
            architecture=self.architecture, vocab_size=V, hidden_size=E, max_positions=self.max_positions,
            embedding=PartSpec("token_embedding", {"vocab_size": V, "hidden_size": E}, {"weight": "embed"}),
            layers=layers, schedule=[ScheduleEntry(layer=i, cache_line=i) for i in range(len(layers))],
            final_norm=norm("final.norm"),
            head=PartSpec("lm_head", {"hidden_size": E, "vocab_size": V}, {"weight": "head"}),
            bos_token_id=None, eos_token_ids=[])
