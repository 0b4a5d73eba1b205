"""Vupolix: a decoder whose sublayers each stand between two norms (a norm in front, a norm of their own
behind, a gain on what they add), with two kinds of mixer in any order: recurrent time mixing with a token
shift, and two mixers side by side, windowed attention with a sink whose values are its unrotated keys
beside retention, each output under a norm of its own.  Feed-forwards are mixtures of experts with a sigmoid
router that chooses within the best groups of experts, and a shared expert.  A stretch of layers runs several
times in a row with the same weights; ahead of every pass but the first the embedding's output, which is a
normed row of the table, is added to the stream again.  The head is a matrix of its own; the logits are
multiplied by a constant.

This file holds what is specific to the design: the keys of its config.json, their checks, the
tensor names of its checkpoints and the translation into a `ModelSpec` of generic parts.

    config.json
      architecture: "Vupolix"; vocab; width; norm.eps; residual_mult; logit_scale; max_positions?
      loop: {start, stop, times}?
      layers: [{type: "wkv", mixer: {heads, dim, rank?}, mlp}
             | {type: "parallel", mixer: {left: {heads, kv_heads, dim, vdim, scale, mask: {size}?, rot?},
                                          right: {heads, dim, vdim, decay: [a number a head], rot?}}, mlp}]
      rot: {base, dims, scaling: {factor, original, fast, slow}?}
      mlp: null | {kind: "moe", expert: {ff}, router: {experts, top, groups: {count, keep}?}, shared: {ff}?}
    tensors
      embed; embed.norm; head; final.norm; l<i>.norm1, .norm1b and, with a feed-forward, .norm2, .norm2b
      wkv (l<i>.mix.): mu.{r, k, v, g, w} [width], r, k, v, g, w1 [rank, width], w2 [heads dim, rank], w0,
                       u [heads, dim], norm [heads dim], o
      parallel: left.{q, k, g [heads, width], sink [heads], o, out [width]}; right.{q, k, v, g, o, out [width]}
      l<i>.mlp.{router, correction, e<j>.{gate, up, down}, shared.{gate, up, down}}

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
# the two outputs of a parallel layer count half each
PAIR_SCALE = 0.5


def _get(d: dict, key: str, where: str, kind=None):
    if not isinstance(d, dict) or key not in d:
        raise ConfigError(f"config.json of Vupolix lacks {where}{key}")
    v = d[key]
    if kind == "int":
        if not isinstance(v, int) or isinstance(v, bool) or v <= 0:
            raise ConfigError(f"{where}{key} must be a positive integer, got {v!r}")
    elif kind in ("float", "number"):
        if isinstance(v, bool) or not isinstance(v, (int, float)) or (kind == "float" and not float(v) > 0):
            raise ConfigError(f"{where}{key} must be a {'positive ' if kind == 'float' else ''}number, got {v!r}")
    return v


def _check_rot(m: dict, at: str) -> None:
    rot = m.get("rot")
    if not rot:
        return
    _get(rot, "base", at + "rot.", "float")
    dims = _get(rot, "dims", at + "rot.", "int")
    if dims % 2 or dims > m["dim"]:
        raise ConfigError(f"{at}rot.dims {dims} must be even and at most dim {m['dim']}")
    if rot.get("scaling"):
        for k in ("factor", "original", "fast", "slow"):
            _get(rot["scaling"], k, at + "rot.scaling.", "float")


def _check_left(m: dict, at: str) -> None:
    for k in ("heads", "kv_heads", "dim", "vdim"):
        _get(m, k, at, "int")
    if m["heads"] % m["kv_heads"]:
        raise ConfigError(f"{at}heads {m['heads']} must be a multiple of kv_heads {m['kv_heads']}")
    if m["vdim"] != m["dim"]:
        raise ConfigError(f"{at}vdim {m['vdim']} must equal dim {m['dim']}: the values are the keys")
    _get(m, "scale", at, "float")
    if m.get("mask"):
        _get(m["mask"], "size", at + "mask.", "int")
    _check_rot(m, at)


def _check_right(m: dict, at: str) -> None:
    for k in ("heads", "dim", "vdim"):
        _get(m, k, at, "int")
    decay = _get(m, "decay", at)
    ok = isinstance(decay, list) and len(decay) == m["heads"] and all(
        isinstance(g, (int, float)) and not isinstance(g, bool) and 0.0 <= float(g) <= 1.0 for g in decay)
    if not ok:
        raise ConfigError(f"{at}decay must list one number in [0, 1] for each of {m['heads']} heads, got {decay!r}")
    _check_rot(m, at)


def _check_mlp(mlp: dict, at: str) -> None:
    if _get(mlp, "kind", at) != "moe":
        raise ConfigError(f"{at}kind {mlp['kind']!r} is not a feed-forward of this design (moe)")
    r = _get(mlp, "router", at)
    n, top = _get(r, "experts", at + "router.", "int"), _get(r, "top", at + "router.", "int")
    most = n
    if r.get("groups"):
        count = _get(r["groups"], "count", at + "router.groups.", "int")
        keep = _get(r["groups"], "keep", at + "router.groups.", "int")
        if n % count or keep > count:
            raise ConfigError(f"{at}router.groups: {keep} of {count} equal groups of {n} experts cannot be kept")
        most = keep * (n // count)
    if top > most:
        raise ConfigError(f"{at}router: {top} of {most} experts cannot be chosen")
    _get(_get(mlp, "expert", at), "ff", at + "expert.", "int")
    if mlp.get("shared"):
        _get(mlp["shared"], "ff", at + "shared.", "int")


@register_architecture("Vupolix")
@dataclass
class VupolixConfig:
    vocab: int
    width: int
    eps: float
    residual_mult: float
    logit_scale: float
    layers: List[dict] = field(default_factory=list)
    loop: Optional[dict] = None
    max_positions: int = DEFAULT_MAX_POSITIONS
    unused_tensors: List[str] = field(default_factory=list)    # in the folder, without a part to act on

    architecture = "Vupolix"
    cli_type_names = ("vupolix",)

    # ------------------------------------------------------------ reading
    @classmethod
    def from_dict(cls, d: dict) -> "VupolixConfig":
        layers = _get(d, "layers", "")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("layers must be a list with at least one layer")
        cfg = cls(vocab=_get(d, "vocab", "", "int"), width=_get(d, "width", "", "int"),
                  eps=float(_get(_get(d, "norm", ""), "eps", "norm.", "float")),
                  residual_mult=float(_get(d, "residual_mult", "", "number")),
                  logit_scale=float(_get(d, "logit_scale", "", "number")), layers=copy.deepcopy(layers),
                  loop=copy.deepcopy(d.get("loop")) or None,
                  max_positions=int(d.get("max_positions", DEFAULT_MAX_POSITIONS)))
        cfg.validate()
        return cfg

    def validate(self) -> None:
        if self.max_positions <= 0:
            raise ConfigError("max_positions must be positive")
        for i, layer in enumerate(self.layers):
            at = f"layers[{i}]."
            kind, m = _get(layer, "type", at), _get(layer, "mixer", at)
            if kind == "wkv":
                for k in ("heads", "dim") + (("rank",) if "rank" in m else ()):
                    _get(m, k, at + "mixer.", "int")
            elif kind == "parallel":
                _check_left(_get(m, "left", at + "mixer."), at + "mixer.left.")
                _check_right(_get(m, "right", at + "mixer."), at + "mixer.right.")
            else:
                raise ConfigError(f"{at}type {kind!r} is not a mixer of this design (wkv, parallel)")
            if layer.get("mlp") is not None:
                _check_mlp(layer["mlp"], at + "mlp.")
        if self.loop is not None:
            start, stop = _get(self.loop, "start", "loop."), _get(self.loop, "stop", "loop.", "int")
            _get(self.loop, "times", "loop.", "int")
            if not isinstance(start, int) or isinstance(start, bool) or not 0 <= start < stop <= len(self.layers):
                raise ConfigError(f"loop: layers {start} .. {stop} - 1 of {len(self.layers)} cannot be repeated")

    def to_dict(self) -> dict:
        d = {"architecture": self.architecture, "layers": copy.deepcopy(self.layers), "logit_scale": self.logit_scale,
             "norm": {"eps": self.eps}, "residual_mult": self.residual_mult, "vocab": self.vocab, "width": self.width}
        if self.loop is not None:
            d["loop"] = copy.deepcopy(self.loop)
        if self.max_positions != DEFAULT_MAX_POSITIONS:
            d["max_positions"] = self.max_positions
        return d

    def with_tensor_shapes(self, shapes: dict) -> "VupolixConfig":
        """The configuration with the sizes that only a folder's tensors state (`shapes`: tensor name
        -> shape): the rank of a wkv layer's decay map.  What a folder holds of a second sublayer that
        the layer does not have is left in the file."""
        cfg = copy.deepcopy(self)
        for i, layer in enumerate(cfg.layers):
            if layer["type"] == "wkv" and f"l{i}.mix.w1" in shapes:
                layer["mixer"]["rank"] = int(shapes[f"l{i}.mix.w1"][0])
            if layer.get("mlp") is None:
                cfg.unused_tensors += [n for n in (f"l{i}.norm2", f"l{i}.norm2b") if n in shapes]
        return cfg

    # ------------------------------------------------------------ translation
    def _rotary(self, m: dict) -> Optional[PartSpec]:
        rot = m.get("rot")
        if not rot:
            return None
        scaling = rot.get("scaling")
        return PartSpec("rotary", {"head_dim": m["dim"], "rotary_dim": int(rot["dims"]), "theta": float(rot["base"]),
                                   "pairing": "half", "max_positions": self.max_positions,
                                   "scaling": ({k: float(scaling[k]) for k in ("factor", "original", "fast", "slow")}
                                               if scaling else None)})

    def _mixer(self, p: str, kind: str, m: dict) -> PartSpec:
        E = self.width
        names = lambda at, *ns: {n: at + n for n in ns}
        if kind == "wkv":
            return PartSpec("time_mix", {"hidden_size": E, "num_heads": m["heads"], "dim": m["dim"],
                                         "decay_rank": int(m.get("rank", DEFAULT_DECAY_RANK)), "eps": self.eps},
                            {**names(p, "r", "k", "v", "g", "w1", "w2", "w0", "u", "norm", "o"),
                             **{f"mu_{s}": f"{p}mu.{s}" for s in ("r", "k", "v", "g", "w")}})
        left, right = m["left"], m["right"]
        attention = PartSpec(
            "gated_attention",
            {"hidden_size": E, "num_heads": left["heads"], "num_kv_heads": left["kv_heads"], "key_dim": left["dim"],
             "value_dim": left["dim"], "softmax_scale": float(left["scale"]),
             "window": int(left["mask"]["size"]) if left.get("mask") else None, "gate": "head", "values": "keys",
             "sink": True}, names(p + "left.", "q", "k", "g", "sink", "o"))
        retention = PartSpec(
            "retention",
            {"hidden_size": E, "num_heads": right["heads"], "key_dim": right["dim"], "value_dim": right["vdim"],
             "decay": [float(g) for g in right["decay"]], "eps": self.eps}, names(p + "right.", "q", "k", "v", "g", "o"))
        return PartSpec("side_by_side",
                        {"left": attention, "right": retention, "left_scale": PAIR_SCALE, "right_scale": PAIR_SCALE,
                         "norm_size": E, "norm_eps": self.eps, "left_position": self._rotary(left),
                         "right_position": self._rotary(right)},
                        {"left_norm": p + "left.out", "right_norm": p + "right.out"})

    def _feed_forward(self, p: str, mlp: Optional[dict]) -> PartSpec:
        if mlp is None:
            return PartSpec("none")
        r, shared = mlp["router"], mlp.get("shared") or None
        groups = r.get("groups") or None
        parts = [f"e{j}" for j in range(int(r["experts"]))] + (["shared"] if shared else [])
        return PartSpec("routed_experts",
                        {"hidden_size": self.width, "expert_size": int(mlp["expert"]["ff"]),
                         "num_experts": int(r["experts"]), "top": int(r["top"]), "score": "sigmoid",
                         "groups": (int(groups["count"]), int(groups["keep"])) if groups else None,
                         "shared_size": int(shared["ff"]) if shared else 0, "shared_gate": False},
                        {"router": p + "router", "correction": p + "correction",
                         **{f"{e}.{t}": f"{p}{e}.{t}" for e in parts for t in ("gate", "up", "down")}})

    def _schedule(self) -> List[ScheduleEntry]:
        """The layers in the order in which they run; every run has a cache line of its own."""
        n, loop = len(self.layers), self.loop or {"start": 0, "stop": 0, "times": 1}
        runs = [(i, False) for i in range(loop["start"])]
        for turn in range(loop["times"]):
            runs += [(i, turn > 0 and i == loop["start"]) for i in range(loop["start"], loop["stop"])]
        runs += [(i, False) for i in range(loop["stop"], n)]
        return [ScheduleEntry(layer=i, cache_line=at, adds_embedding=again) for at, (i, again) in enumerate(runs)]

    def to_spec(self) -> ModelSpec:
        E, V = self.width, self.vocab
        norm = lambda name, **kw: PartSpec("rms_norm", {"size": E, "eps": self.eps, **kw}, {"weight": name})
        layers = []
        for i, layer in enumerate(self.layers):
            mlp = layer.get("mlp")
            own = {"post1": f"l{i}.norm1b"} | ({"post2": f"l{i}.norm2b"} if mlp is not None else {})
            layers.append(LayerSpec(
                block="sandwich", mixer=self._mixer(f"l{i}.mix.", layer["type"], layer["mixer"]),
                feed_forward=self._feed_forward(f"l{i}.mlp.", mlp), mixer_norm=norm(f"l{i}.norm1"),
                feed_forward_norm=norm(f"l{i}.norm2") if mlp is not None else None,
                block_params={"size": E, "eps": self.eps, "gain": self.residual_mult}, block_tensors=own))
        return ModelSpec(
            architecture=self.architecture, vocab_size=V, hidden_size=E, max_positions=self.max_positions,
            embedding=PartSpec("token_embedding", {"vocab_size": V, "hidden_size": E, "norm_eps": self.eps},
                               {"weight": "embed", "norm": "embed.norm"}),
            layers=layers, schedule=self._schedule(), final_norm=norm("final.norm", scale=self.logit_scale),
            head=PartSpec("lm_head", {"hidden_size": E, "vocab_size": V}, {"weight": "head"}),
            bos_token_id=None, eos_token_ids=[], ignored_tensor_suffixes=list(self.unused_tensors))
