"""Typed configuration of the Tokatar architecture, read from config.json.

A Tokatar model is a list of layers around one float32 residual stream.  Every sublayer f (a mixer, then a feed-forward
unless the layer has none) is wrapped the same way: with u = norm(x), the stream becomes
x + ls * norm(sigmoid(R u + b) * f(u)): a norm before it, a gate computed from its input, a norm behind it (every norm's
weight is ONE number) and a vector of scales.  Three mixers:

* ``attention``: grouped-query softmax attention with rotary positions (pairs of halves, optionally llama3-scaled),
  scores capped by a tanh, keys of the query's own chunk of positions only, a sigmoid gate on the heads;
* ``attention_2``: the same with biases on q, k and v, a norm over the whole q and the whole k projection, pairs of
  neighbours, values turned by their positions (and outputs turned back), one added to the softmax's denominator;
* ``latent_attention``: causal softmax attention whose keys and values are linear maps of one normed latent a token,
  beside one rotated key part that all heads share, a sigmoid gate of one number per head.

The feed-forward is ungated, with the square of ReLU.  The embedding multiplies the token's row by ``embedding.scale``.

config.json keys: ``architecture``, ``vocab``, ``width``, ``norm.eps``, ``embedding.scale`` and ``layers`` (a list of
``{"type", "mixer": {...}, "mlp": {...} or null}``).  Tensor names: ``embed``, ``head``, ``final.norm`` and per layer i
``l<i>.norm1``, ``norm1b``, ``ls1``, ``rg1``, ``rg1.b`` (and the same with 2 for the feed-forward), ``mix.*``, ``mlp.*``.
"""
from __future__ import annotations

import json
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from .bomotar import DEFAULT_MAX_POSITIONS, _obj
from .llama import ConfigError
from .mifutar import _num
from .spec import LayerCall, LayerSpec, ModelSpec, PartSpec

#: the feed-forward's activation and the score of ``attention_2``'s sink (e^0 = 1 in the denominator), fixed by the design
ACTIVATION = "relu2"
SINK_SCORE = 0.0
#: which elements of a head turn together, by mixer type
ROTARY_LAYOUT = {"attention": "halves", "attention_2": "neighbours", "latent_attention": "halves"}
MIXERS = tuple(ROTARY_LAYOUT)


@dataclass(frozen=True)
class Scaling:
    factor: float
    low: float
    high: float
    original: float

    def to_dict(self):
        return {"factor": self.factor, "high": self.high, "low": self.low, "original": self.original}


@dataclass(frozen=True)
class Rotation:
    dims: int
    base: float
    scaling: Optional[Scaling] = None

    @classmethod
    def from_dict(cls, d, where, most):
        s = _obj(d, "scaling", where, optional=True)
        if s is not None:
            s = Scaling(*(_num(s, key, where + ".scaling", float) for key in ("factor", "low", "high", "original")))
            if s.high < s.low:
                raise ConfigError(f"config.json: {where}.scaling: high ({s.high:g}) below low ({s.low:g})")
        r = cls(_num(d, "dims", where) if d.get("dims") is not None else most, _num(d, "base", where, float), s)
        if r.dims % 2 != 0 or r.dims > most:
            raise ConfigError(f"config.json: {where}: dims ({r.dims}) must be even and at most {most}")
        return r

    def to_dict(self):
        d = {"base": self.base, "dims": self.dims}
        if self.scaling is not None:
            d["scaling"] = self.scaling.to_dict()
        return d

    def part(self, head_dim: int, layout: str) -> PartSpec:
        scaling = None
        if self.scaling is not None:
            s = self.scaling
            scaling = {"rope_type": "llama3", "factor": s.factor, "low_freq_factor": s.low, "high_freq_factor": s.high,
                       "original_max_position_embeddings": s.original}
        return PartSpec("rope", {"head_dim": head_dim, "rotary_dim": self.dims, "theta": self.base, "scaling": scaling, "layout": layout})


@dataclass(frozen=True)
class AttentionMixer:
    """``attention`` and ``attention_2``."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Rotation
    chunk: Optional[int] = None
    softcap: Optional[float] = None

    @classmethod
    def from_dict(cls, d, where):
        mask = _obj(d, "mask", where, optional=True)
        heads, dim = _num(d, "heads", where), _num(d, "dim", where)
        m = cls(heads, _num(d, "kv_heads", where) if d.get("kv_heads") is not None else heads, dim,
                _num(d, "vdim", where) if d.get("vdim") is not None else dim, _num(d, "scale", where, float),
                Rotation.from_dict(_obj(d, "rot", where), where + ".rot", dim),
                None if mask is None else _num(mask, "size", where + ".mask"),
                None if d.get("softcap") is None else _num(d, "softcap", where, float))
        if m.heads % m.kv_heads != 0:
            raise ConfigError(f"config.json: {where}: heads ({m.heads}) must be a multiple of kv_heads ({m.kv_heads})")
        if m.dim % 2 != 0 or m.vdim % 2 != 0:
            raise ConfigError(f"config.json: {where}: dim ({m.dim}) and vdim ({m.vdim}) must be even")
        return m

    def to_dict(self):
        d = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "rot": self.rot.to_dict(), "scale": self.scale, "vdim": self.vdim}
        if self.chunk is not None:
            d["mask"] = {"size": self.chunk}
        if self.softcap is not None:
            d["softcap"] = self.softcap
        return d


@dataclass(frozen=True)
class LatentMixer:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot: Rotation

    @classmethod
    def from_dict(cls, d, where):
        dim, rot_dim = _num(d, "dim", where), _num(d, "rot_dim", where)
        m = cls(_num(d, "heads", where), dim, rot_dim, _num(d, "vdim", where) if d.get("vdim") is not None else dim,
                _num(d, "kv_rank", where), _num(d, "scale", where, float), Rotation.from_dict(_obj(d, "rot", where), where + ".rot", rot_dim))
        if m.rot.dims != rot_dim:
            raise ConfigError(f"config.json: {where}: rot.dims ({m.rot.dims}) must be rot_dim ({rot_dim})")
        if m.kv_rank % 2 != 0:
            raise ConfigError(f"config.json: {where}: kv_rank ({m.kv_rank}) must be even")
        return m

    def to_dict(self):
        return {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank, "rot": self.rot.to_dict(), "rot_dim": self.rot_dim,
                "scale": self.scale, "vdim": self.vdim}


@dataclass(frozen=True)
class DenseMlp:
    ff: int

    def to_dict(self):
        return {"ff": self.ff, "kind": "dense"}


@dataclass(frozen=True)
class TokatarLayer:
    type: str
    mixer: Any                  # AttentionMixer or LatentMixer
    mlp: Optional[DenseMlp]


@dataclass
class TokatarConfig:
    vocab: int
    width: int
    layers: List[TokatarLayer]
    embedding_scale: float = 1.0
    norm_eps: float = 1e-6
    max_positions: int = DEFAULT_MAX_POSITIONS
    eos_token_id: List[int] = field(default_factory=list)
    architecture: str = "Tokatar"

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
    def from_dict(cls, d: Dict[str, Any]) -> "TokatarConfig":
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
            md = _obj(ld, "mixer", where)
            mixer = (LatentMixer if kind == "latent_attention" else AttentionMixer).from_dict(md, where + ".mixer")
            mlp = _obj(ld, "mlp", where, optional=True)
            if mlp is not None:
                if mlp.get("kind", "dense") != "dense":
                    raise ConfigError(f"config.json: {where}.mlp: feed-forward kind {mlp.get('kind')!r} unknown (known: dense)")
                mlp = DenseMlp(_num(mlp, "ff", where + ".mlp"))
            layers.append(TokatarLayer(kind, mixer, mlp))
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
            architecture=str(d.get("architecture", "Tokatar")),
        )

    @classmethod
    def from_json(cls, text: str) -> "TokatarConfig":
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
                n *= int(s)
            total += n
        return total

    def kv_bytes_per_token(self, elem_bytes: int = 2) -> int:
        """What a token's keys and values are (pages may pad them; a chunked layer gives finished chunks back)."""
        total = 0
        for l in self.layers:
            m = l.mixer
            total += (m.rot_dim + 2 * m.kv_rank if l.type == "latent_attention" else m.kv_heads * (m.dim + m.vdim)) * elem_bytes
        return total

    def describe(self) -> Dict[str, Any]:
        """What ``tempura inspect`` prints of this architecture."""
        def layer(l):
            m = l.mixer
            if l.type == "latent_attention":
                mix = f"latent attention {m.heads} heads of {m.dim} and {m.rot_dim} rotated, values of {m.vdim}, latent {m.kv_rank}, gate per head"
            else:
                mix = f"{l.type} {m.heads} heads ({m.kv_heads} key/value) of {m.dim}, values of {m.vdim}, " + \
                    ("no chunks" if m.chunk is None else f"chunks of {m.chunk}") + f", {m.rot.dims} rotated" + \
                    ("" if m.softcap is None else f", scores capped at {m.softcap:g}") + \
                    (", biases, norm over the projection, turned values, one in the denominator" if l.type == "attention_2" else "") + ", gate"
            return mix + ("; no feed-forward" if l.mlp is None else f"; feed-forward {l.mlp.ff}")
        return {"hidden_size": self.width, "vocab_size": self.vocab, "norm_eps": self.norm_eps, "max_positions": self.max_positions,
                "embedding_scale": self.embedding_scale, "layers": [layer(l) for l in self.layers],
                "kv_bytes_per_token_bf16": self.kv_bytes_per_token(2)}

    def _mixer(self, kind: str, m, p: str) -> PartSpec:
        layout = ROTARY_LAYOUT[kind]
        if kind == "latent_attention":
            return PartSpec(
                "rotary_latent_attention",
                params={"num_heads": m.heads, "head_dim": m.dim, "rotary_dim": m.rot_dim, "value_dim": m.vdim, "latent_dim": m.kv_rank,
                        "scale": m.scale, "norm_eps": self.norm_eps, "gate": "head", "position": m.rot.part(m.rot_dim, layout)},
                weights={"q": f"{p}.q", "dkv": f"{p}.dkv", "dkv_norm": f"{p}.dkv.norm", "uk": f"{p}.uk", "uv": f"{p}.uv", "gate": f"{p}.g",
                         "o": f"{p}.o"})
        params = {"num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim, "value_dim": m.vdim, "scale": m.scale,
                  "chunk": m.chunk, "softcap": m.softcap, "gate": True, "position": m.rot.part(m.dim, layout)}
        weights = {"q": f"{p}.q", "k": f"{p}.k", "v": f"{p}.v", "gate": f"{p}.g", "o": f"{p}.o"}
        if kind == "attention_2":
            params.update({"bias": True, "qk_norm": {"eps": self.norm_eps, "over": "projection"}, "sink": SINK_SCORE,
                           "value_position": Rotation(m.vdim, m.rot.base).part(m.vdim, layout)})
            weights.update({"q_bias": f"{p}.q.b", "k_bias": f"{p}.k.b", "v_bias": f"{p}.v.b", "q_norm": f"{p}.q.norm", "k_norm": f"{p}.k.norm"})
        return PartSpec("attention", params, weights)

    def build_spec(self) -> ModelSpec:
        norm = lambda name: PartSpec("rmsnorm", {"eps": self.norm_eps, "scalar": True}, {"weight": name})
        layers = []
        for i, l in enumerate(self.layers):
            p = f"l{i}"
            parts = {"mixer": self._mixer(l.type, l.mixer, f"{p}.mix")}
            if l.mlp is not None:
                parts["ffn"] = PartSpec("mlp", {"intermediate_size": l.mlp.ff, "activation": ACTIVATION},
                                        {"up": f"{p}.mlp.up", "down": f"{p}.mlp.down"})
            for n, name in ((1, "mixer"), (2, "ffn")):
                if name in parts:
                    parts.update({name + "_norm": norm(f"{p}.norm{n}"), name + "_post_norm": norm(f"{p}.norm{n}b"),
                                  name + "_gate": PartSpec("input_sigmoid", {}, {"weight": f"{p}.rg{n}", "bias": f"{p}.rg{n}.b"}),
                                  name + "_scale": PartSpec("vector", {}, {"weight": f"{p}.ls{n}"})})
            layers.append(LayerSpec("sandwich", parts))
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
