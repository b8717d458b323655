"""Typed configuration of the Makisun architecture, read from config.json.

A Makisun model is a list of layers around one float32 residual stream; a layer is x <- x + ls1 * mixer(norm1(x)), then,
unless it has no feed-forward, x <- x + ls2 * ff(norm2(x)): RMS norms whose weights are stored around zero, and a vector
of scales on what each sublayer adds.  Two mixers:

* ``wkv``: a linear recurrence with a decay per key channel that depends on the token, whose five projections each read
  their own mix of a token's normed row and the row before it, with a bonus for the current token;
* ``parallel``: two mixers on the same input, added with ``left_scale`` and ``right_scale``: a grouped-query softmax
  attention (a norm per head on q and k, rotary positions on part of a head, a sliding window, a sigmoid gate of one
  number per head) and a gated linear attention (a decay per key channel, sigmoid(z)^(1/tau)).

Feed-forwards: ``dense`` (ungated, the exact GELU) or ``moe`` (ungated experts with the square of ReLU, a router with a
bias whose weights are a softmax over the chosen logits, optionally a shared expert that every token uses).  The embedding
multiplies the token's row by ``embedding.scale``.

config.json keys: ``architecture``, ``vocab``, ``width``, ``norm.eps``, ``embedding.scale`` and ``layers`` (a list of
``{"type", "mixer": {...}, "mlp": {...} or null}``).  Tensor names: ``embed``, ``head``, ``final.norm`` and per layer i
``l<i>.norm1``, ``l<i>.ls1`` (and the same with 2 for the feed-forward), ``l<i>.mix.*``, ``l<i>.mlp.*``.
"""
from __future__ import annotations

import json
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from .bomotar import DEFAULT_MAX_POSITIONS, Rotation, _obj
from .llama import ConfigError
from .mifutar import _num
from .spec import LayerCall, LayerSpec, ModelSpec, PartSpec

#: activations of the dense feed-forward and of an expert, routed or shared (fixed by the design)
DENSE_ACTIVATION = "gelu_erf"
EXPERT_ACTIVATION = "relu2"
#: the weight of every norm of a layer and of the model's last norm is stored as its deviation from one
NORM_WEIGHT_OFFSET = 1.0
MIXERS = ("wkv", "parallel")


def _rank(d, key, where) -> Optional[int]:
    """The inner size of a low-rank projection: the checkpoint's tensors say it; a configuration names it only where no
    checkpoint is there to say it, for random weights."""
    return _num(d, key, where) if d.get(key) is not None else None


@dataclass(frozen=True)
class WkvMixer:
    heads: int
    dim: int
    decay_rank: Optional[int] = None

    @classmethod
    def from_dict(cls, d, where):
        return cls(_num(d, "heads", where), _num(d, "dim", where), _rank(d, "decay_rank", where))

    def to_dict(self):
        d = {"dim": self.dim, "heads": self.heads}
        if self.decay_rank is not None:
            d["decay_rank"] = self.decay_rank
        return d


@dataclass(frozen=True)
class LeftMixer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Optional[Rotation]
    window: Optional[int] = None

    @classmethod
    def from_dict(cls, d, where):
        heads, dim = _num(d, "heads", where), _num(d, "dim", where)
        rot, mask = _obj(d, "rot", where, optional=True), _obj(d, "mask", where, optional=True)
        if rot is not None and rot.get("dims") is None:
            rot = dict(rot, dims=dim)
        m = cls(heads, _num(d, "kv_heads", where) if d.get("kv_heads") is not None else heads, dim,
                _num(d, "vdim", where) if d.get("vdim") is not None else dim, _num(d, "scale", where, float),
                None if rot is None else Rotation.from_dict(rot, where + ".rot", dim),
                None if mask is None else _num(mask, "size", where + ".mask"))
        if m.heads % m.kv_heads != 0:
            raise ConfigError(f"config.json: {where}: heads ({m.heads}) must be a multiple of kv_heads ({m.kv_heads})")
        return m

    def to_dict(self):
        d = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale, "vdim": self.vdim}
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        if self.window is not None:
            d["mask"] = {"size": self.window}
        return d


@dataclass(frozen=True)
class RightMixer:
    heads: int
    dim: int
    vdim: int
    tau: float
    decay_rank: Optional[int] = None

    @classmethod
    def from_dict(cls, d, where):
        dim = _num(d, "dim", where)
        return cls(_num(d, "heads", where), dim, _num(d, "vdim", where) if d.get("vdim") is not None else dim,
                   _num(d, "tau", where, float), _rank(d, "decay_rank", where))

    def to_dict(self):
        d = {"dim": self.dim, "heads": self.heads, "tau": self.tau, "vdim": self.vdim}
        if self.decay_rank is not None:
            d["decay_rank"] = self.decay_rank
        return d


@dataclass(frozen=True)
class ParallelMixerConfig:
    left: LeftMixer
    right: RightMixer
    left_scale: float
    right_scale: float

    @classmethod
    def from_dict(cls, d, where):
        return cls(LeftMixer.from_dict(_obj(d, "left", where), where + ".left"), RightMixer.from_dict(_obj(d, "right", where), where + ".right"),
                   _num(d, "left_scale", where, float, positive=False), _num(d, "right_scale", where, float, positive=False))

    def to_dict(self):
        return {"left": self.left.to_dict(), "left_scale": self.left_scale, "right": self.right.to_dict(), "right_scale": self.right_scale}


@dataclass(frozen=True)
class DenseMlp:
    ff: int

    def to_dict(self):
        return {"ff": self.ff, "kind": "dense"}


@dataclass(frozen=True)
class MoeMlp:
    ff: int
    experts: int
    top: int
    shared_ff: Optional[int] = None

    def to_dict(self):
        d = {"expert": {"ff": self.ff}, "kind": "moe", "router": {"experts": self.experts, "top": self.top}}
        if self.shared_ff is not None:
            d["shared"] = {"ff": self.shared_ff}
        return d


def _mlp_from_dict(d, where):
    kind = d.get("kind", "dense")
    if kind == "dense":
        return DenseMlp(_num(d, "ff", where))
    if kind == "moe":
        r = _obj(d, "router", where)
        sh = _obj(d, "shared", where, optional=True)
        m = MoeMlp(_num(_obj(d, "expert", where), "ff", where + ".expert"), _num(r, "experts", where + ".router"), _num(r, "top", where + ".router"),
                   None if sh is None else _num(sh, "ff", where + ".shared"))
        if m.top > m.experts:
            raise ConfigError(f"config.json: {where}.router: top ({m.top}) exceeds experts ({m.experts})")
        return m
    raise ConfigError(f"config.json: {where}: feed-forward kind {kind!r} unknown (known: dense, moe)")


@dataclass(frozen=True)
class MakisunLayer:
    type: str
    mixer: Any      # WkvMixer or ParallelMixerConfig
    mlp: Any        # DenseMlp, MoeMlp or None


@dataclass
class MakisunConfig:
    vocab: int
    width: int
    layers: List[MakisunLayer]
    embedding_scale: float = 1.0
    norm_eps: float = 1e-6
    max_positions: int = DEFAULT_MAX_POSITIONS
    eos_token_id: List[int] = field(default_factory=list)
    architecture: str = "Makisun"

    # (names the engine's reports and sizing read from any configuration)
    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @property
    def max_position_embeddings(self) -> int:
        return self.max_positions

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "MakisunConfig":
        layers_in = d.get("layers")
        if not isinstance(layers_in, list) or not layers_in:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        layers = []
        for i, ld in enumerate(layers_in):
            where = f"layers[{i}]"
            if not isinstance(ld, dict):
                raise ConfigError(f"config.json: {where} must be an object")
            kind = ld.get("type")
            if kind not in MIXERS:
                raise ConfigError(f"config.json: {where}: mixer type {kind!r} unknown (known: {', '.join(MIXERS)})")
            mixer = (WkvMixer if kind == "wkv" else ParallelMixerConfig).from_dict(_obj(ld, "mixer", where), where + ".mixer")
            mlp = None if ld.get("mlp") is None else _mlp_from_dict(_obj(ld, "mlp", where), where + ".mlp")
            layers.append(MakisunLayer(kind, mixer, mlp))
        norm = d.get("norm") or {}
        if not isinstance(norm, dict):
            raise ConfigError("config.json: 'norm' must be an object")
        emb = _obj(d, "embedding", "top level", optional=True) or {}
        eos = d.get("eos_token_id")
        return cls(
            vocab=_num(d, "vocab", "top level"),
            width=_num(d, "width", "top level"),
            layers=layers,
            embedding_scale=_num(emb, "scale", "embedding", float, positive=False) if emb.get("scale") is not None else 1.0,
            norm_eps=_num(norm, "eps", "norm", float) if norm.get("eps") is not None else 1e-6,
            max_positions=_num(d, "max_positions", "top level") if d.get("max_positions") is not None else DEFAULT_MAX_POSITIONS,
            eos_token_id=[] if eos is None else ([int(e) for e in eos] if isinstance(eos, list) else [int(eos)]),
            architecture=str(d.get("architecture", "Makisun")),
        )

    @classmethod
    def from_json(cls, text: str) -> "MakisunConfig":
        try:
            d = json.loads(text)
        except json.JSONDecodeError as e:
            raise ConfigError(f"config.json: malformed JSON: {e}") from e
        if not isinstance(d, dict):
            raise ConfigError("config.json: top level must be an object")
        return cls.from_dict(d)

    def to_dict(self) -> Dict[str, Any]:
        d = {
            "architecture": self.architecture,
            "embedding": {"scale": self.embedding_scale},
            "layers": [{"mixer": l.mixer.to_dict(), "mlp": None if l.mlp is None else l.mlp.to_dict(), "type": l.type} for l in self.layers],
            "norm": {"eps": self.norm_eps},
            "vocab": self.vocab,
            "width": self.width,
        }
        if self.max_positions != DEFAULT_MAX_POSITIONS:
            d["max_positions"] = self.max_positions
        if self.eos_token_id:
            d["eos_token_id"] = list(self.eos_token_id)
        return d

    def to_json(self) -> str:
        return json.dumps(self.to_dict(), indent=1)

    # ---- derived ---------------------------------------------------------
    def num_parameters(self) -> int:
        from ..parts.inventory import expected_weights
        total = 0
        for info in expected_weights(self.build_spec()).values():
            n = 1
            for s in info.shape:
                n *= int(s) if s is not None else 0      # (a size only the checkpoint says: not counted)
            total += n
        return total

    def kv_bytes_per_token(self, elem_bytes: int = 2) -> int:
        """What a token's keys and values are (a windowed layer gives pages behind the window back)."""
        return sum(l.mixer.left.kv_heads * (l.mixer.left.dim + l.mixer.left.vdim) * elem_bytes for l in self.layers if l.type == "parallel")

    def state_bytes_per_request(self) -> int:
        total = 0
        for l in self.layers:
            if l.type == "wkv":
                total += 4 * (l.mixer.heads * l.mixer.dim * l.mixer.dim + self.width)      # the state and the row before
            else:
                total += 4 * l.mixer.right.heads * l.mixer.right.dim * l.mixer.right.vdim
        return total

    def describe(self) -> Dict[str, Any]:
        """What ``tempura inspect`` prints of this architecture."""
        def layer(l):
            m = l.mixer
            if l.type == "wkv":
                mix = f"wkv {m.heads} heads of {m.dim}"
            else:
                a, r = m.left, m.right
                mix = (f"{m.left_scale:g} x attention {a.heads} heads ({a.kv_heads} key/value) of {a.dim}, values of {a.vdim}, "
                       + ("no window" if a.window is None else f"window {a.window}") + ", "
                       + ("no rotation" if a.rot is None else f"{a.rot.dims} rotated") + ", gate per head"
                       + f" + {m.right_scale:g} x gated linear attention {r.heads} heads of {r.dim}, values of {r.vdim}, tau {r.tau:g}")
            if l.mlp is None:
                ff = "no feed-forward"
            elif isinstance(l.mlp, DenseMlp):
                ff = f"feed-forward {l.mlp.ff}"
            else:
                ff = f"{l.mlp.experts} experts of {l.mlp.ff}, {l.mlp.top} a token" + \
                    (f", shared expert of {l.mlp.shared_ff}" if l.mlp.shared_ff is not None else "")
            return mix + "; " + ff
        return {"hidden_size": self.width, "vocab_size": self.vocab, "norm_eps": self.norm_eps, "max_positions": self.max_positions,
                "embedding_scale": self.embedding_scale, "layers": [layer(l) for l in self.layers],
                "kv_bytes_per_token_bf16": self.kv_bytes_per_token(2), "state_bytes_per_request": self.state_bytes_per_request()}

    def _mixer(self, kind: str, m, p: str) -> PartSpec:
        if kind == "wkv":
            names = {name: f"{p}.{name}" for name in ("r", "k", "v", "w1", "w2", "w0", "u", "norm", "o")}
            return PartSpec(
                "wkv",
                params={"num_heads": m.heads, "head_dim": m.dim, "norm_eps": self.norm_eps, "decay_rank": m.decay_rank},
                weights=dict(names, gate=f"{p}.g", **{"mu_" + s: f"{p}.mu.{s}" for s in ("r", "k", "v", "g", "w")}))
        a, r = m.left, m.right
        left = PartSpec(
            "branch_attention",
            params={"num_heads": a.heads, "num_kv_heads": a.kv_heads, "head_dim": a.dim, "value_dim": a.vdim, "scale": a.scale,
                    "window": a.window, "gate": "head", "qk_norm": {"eps": self.norm_eps},
                    "position": PartSpec("none") if a.rot is None else a.rot.part(a.dim)},
            weights={"q": f"{p}.left.q", "k": f"{p}.left.k", "v": f"{p}.left.v", "q_norm": f"{p}.left.q.norm", "k_norm": f"{p}.left.k.norm",
                     "gate": f"{p}.left.g", "o": f"{p}.left.o"})
        right = PartSpec(
            "gated_linear",
            params={"num_heads": r.heads, "head_dim": r.dim, "value_dim": r.vdim, "q_scale": r.dim ** -0.5, "decay_root": r.tau,
                    "norm_eps": self.norm_eps, "decay_rank": r.decay_rank},
            weights={"q": f"{p}.right.q", "k": f"{p}.right.k", "v": f"{p}.right.v", "gate": f"{p}.right.g", "o": f"{p}.right.o",
                     "norm": f"{p}.right.norm", "a1": f"{p}.right.a1", "a2": f"{p}.right.a2", "a2_bias": f"{p}.right.a2.b"})
        return PartSpec("parallel", params={"branches": [left, right], "scales": [m.left_scale, m.right_scale]})

    def _ffn(self, mlp, p: str) -> PartSpec:
        if isinstance(mlp, DenseMlp):
            return PartSpec("mlp", {"intermediate_size": mlp.ff, "activation": DENSE_ACTIVATION}, {"up": f"{p}.up", "down": f"{p}.down"})
        params = {"experts": mlp.experts, "top": mlp.top, "intermediate_size": mlp.ff, "expert": "plain", "activation": EXPERT_ACTIVATION,
                  "normalize": True, "sum_eps": 0.0}
        weights = {"router": f"{p}.router", "router_bias": f"{p}.router.b", "up": p + ".e{}.up", "down": p + ".e{}.down"}
        if mlp.shared_ff is not None:
            params["shared"] = {"intermediate_size": mlp.shared_ff, "activation": EXPERT_ACTIVATION}
            weights.update({"shared_up": f"{p}.shared.up", "shared_down": f"{p}.shared.down"})
        return PartSpec("moe", params, weights)

    def build_spec(self) -> ModelSpec:
        norm = lambda name: PartSpec("rmsnorm", {"eps": self.norm_eps, "weight_offset": NORM_WEIGHT_OFFSET}, {"weight": name})
        layers = []
        for i, l in enumerate(self.layers):
            p = f"l{i}"
            parts = {"mixer": self._mixer(l.type, l.mixer, f"{p}.mix")}
            if l.mlp is not None:
                parts["ffn"] = self._ffn(l.mlp, f"{p}.mlp")
            for n, name in ((1, "mixer"), (2, "ffn")):
                if name in parts:
                    parts[name + "_norm"] = norm(f"{p}.norm{n}")
                    parts[name + "_scale"] = PartSpec("vector", {}, {"weight": f"{p}.ls{n}"})
            layers.append(LayerSpec("scaled_prenorm", parts))
        return ModelSpec(
            architecture=self.architecture,
            hidden_size=self.width,
            vocab_size=self.vocab,
            max_positions=self.max_positions,
            layers=layers,
            order=[LayerCall(i) for i in range(len(layers))],
            final_norm=norm("final.norm"),
            embedding=PartSpec("embedding", {"scale": self.embedding_scale}, {"weight": "embed"}),
            lm_head=PartSpec("lm_head", {"tied": False}, {"weight": "head"}),
            eos_token_ids=list(self.eos_token_id),
        )
