"""Litizen as data: its config.json typed, and turned into a `ModelSpec`.

A decoder-only model whose layers are listed one by one in config.json (`layers`: each entry a `type`, the mixer's sizes
under `mixer`, and `mlp` or null).  What the design fixes is written here; what config.json gives is read from there:

  embedding   x = embed[token] * embedding.scale
  layer i     x <- x + norm1b(mixer(h + conv(h))), h = norm1(x); then x <- x + norm2b(ff(norm2(x))); `mlp: null` leaves the
              second out.  Every model norm divides norm.groups equal parts of the row by their own root mean squares and
              multiplies by a weight as long as the row (block "sandwich"); conv is causal, a weight a channel and tap,
              over the last canon.taps inputs (`parts/short_conv.py`)
  type "attention"    grouped-query softmax attention over the last mask.size tokens whose values are the keys as projected;
              q and k RMS-normed head by head with a weight, then turned on their first rot.dims dims in pairs
              (i, i + rot.dims / 2); score (q . k) * scale; one added to every softmax's denominator; the heads times
              sigmoid(g h) before `o`
  type "attention_2"  grouped-query softmax attention within chunks of mask.size positions; q and k turned the same way, values
              turned over all their dims by their own positions and the result turned back by the query's; score softcap *
              tanh((q . k) * scale / softcap); exp(sink) of the head in the denominator; the same gate
  type "mamba2"       a selective state space per head with a short causal convolution in front, a gate and a grouped RMS
              norm behind (`parts/ssm.py`)
  mlp         dense: down(silu(gate h) * (up h)); moe: `router.experts` such feed-forwards of `expert.ff` and `router.identity`
              experts that return their input; a token takes the `router.top` with the largest softmax score + correction,
              weighted by their scores over the scores' sum; with `shared` one more of `shared.ff` that every token takes
  output      the norm `final.norm`, `head`, logit_softcap * tanh(logits / logit_softcap)

Tensor names: `embed`, `l<i>.{norm1,norm1b,norm2,norm2b}`, `l<i>.canon1`, `l<i>.mix.*`, `l<i>.mlp.{gate,up,down}` or
`l<i>.mlp.{router,correction,e<j>.*,shared.*}`, `final.norm`, `head`.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from ..config.model_config import ConfigError, _require
from ..config.spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry
from .debusun import DEFAULT_POSITIONS, Rotary, StateSpaceMixer, _obj, _opt, _window
from .registry import ModelFamily, register_architecture


@dataclass(frozen=True)
class _Attention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    span: int                          # mask.size; 0: every earlier token is seen
    rot: Optional[Rotary]
    softcap: Optional[float] = None

    @classmethod
    def from_dict(cls, raw: Any, where: str) -> "_Attention":
        raw = _obj(raw, "mixer", where)
        dim = _require(raw, "dim", int, where)
        m = cls(_require(raw, "heads", int, where), _require(raw, "kv_heads", int, where), dim, _opt(raw, "vdim", int, where) or dim,
                _require(raw, "scale", float, where), _window(raw, where),
                Rotary.from_dict(raw["rot"], where) if raw.get("rot") is not None else None, _opt(raw, "softcap", float, where))
        if min(m.heads, m.kv_heads, m.dim, m.vdim) <= 0 or m.heads % m.kv_heads:
            raise ConfigError(f"{where}: {m.heads} heads of {m.dim}/{m.vdim} on {m.kv_heads} kv heads cannot be run")
        if m.rot is not None and (m.rot.dims > m.dim or m.rot.scaling is not None):
            raise ConfigError(f"{where}: rot turns at most a head's {m.dim} dims, without scaling")
        if m.softcap is not None and not m.softcap > 0:
            raise ConfigError(f"{where}: softcap must be positive or absent")
        m.check(where)
        return m

    def check(self, where: str) -> None:
        pass

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.span:
            out["mask"] = {"size": self.span}
        if self.rot is not None:
            out["rot"] = self.rot.to_dict()
        if self.softcap is not None:
            out["softcap"] = self.softcap
        return out

    def common(self, cfg: "LitizenConfig") -> Dict[str, Any]:
        return dict(hidden_size=cfg.width, num_heads=self.heads, num_kv_heads=self.kv_heads, head_dim=self.dim, value_dim=self.vdim,
                    bias=False, scale=self.scale, score_softcap=self.softcap, gate=True, general=True,
                    position=None if self.rot is None else self.turn(self.rot.dims, self.dim, cfg),
                    names={"q": "q", "k": "k", "v": "v", "o": "o", "gate": "g", "q_norm": "q.norm", "k_norm": "k.norm", "sink": "sink"})

    def turn(self, dims: int, head: int, cfg: "LitizenConfig") -> PartSpec:
        p = Rotary(dims, self.rot.base).spec(head, cfg.max_positions, interleaved=False)
        return PartSpec(p.kind, dict(p.params, precise=True))


@dataclass(frozen=True)
class KeyValueAttention(_Attention):
    """type "attention"."""

    def check(self, where: str) -> None:
        if self.vdim != self.dim:
            raise ConfigError(f"{where}: values that are the keys have the keys' {self.dim} dims, not {self.vdim}")

    def spec(self, cfg: "LitizenConfig") -> PartSpec:
        return PartSpec("attention", dict(self.common(cfg), values="keys", qk_norm=True, qk_norm_eps=cfg.norm_eps,
                                          window=self.span or None, sinks="one"))


@dataclass(frozen=True)
class TurnedValueAttention(_Attention):
    """type "attention_2"."""

    def check(self, where: str) -> None:
        if self.rot is not None and self.vdim % 2:
            raise ConfigError(f"{where}: values of {self.vdim} dims do not turn in pairs")

    def spec(self, cfg: "LitizenConfig") -> PartSpec:
        return PartSpec("attention", dict(self.common(cfg), qk_norm=False, window=None, chunk=self.span, sinks="learned",
                                          value_position=None if self.rot is None else self.turn(self.vdim, self.vdim, cfg)))


@dataclass(frozen=True)
class StateSpace(StateSpaceMixer):
    """type "mamba2"."""

    def spec(self, cfg: "LitizenConfig") -> PartSpec:
        return PartSpec("mamba2", dict(hidden_size=cfg.width, num_heads=self.heads, value_dim=self.vdim, state_dim=self.state,
                                       groups=self.groups, conv=self.conv, norm_groups=self.norm_groups, norm_eps=cfg.norm_eps))


MIXERS = {"attention": KeyValueAttention, "attention_2": TurnedValueAttention, "mamba2": StateSpace}


@dataclass(frozen=True)
class FeedForward:
    kind: str                          # "dense" or "moe"
    ff: int                            # inner size of the dense feed-forward, or of an expert
    experts: int = 0
    top: int = 0
    identity: int = 0
    shared: int = 0                    # inner size of the shared expert; 0: none

    @classmethod
    def from_dict(cls, raw: Any, where: str) -> "FeedForward":
        raw = _obj(raw, "mlp", where)
        kind = str(raw.get("kind", "dense"))
        if kind == "dense":
            f = cls("dense", _require(raw, "ff", int, where))
        elif kind == "moe":
            r = _obj(raw.get("router"), "mlp.router", where)
            shared = raw.get("shared")
            f = cls("moe", _require(_obj(raw.get("expert"), "mlp.expert", where), "ff", int, where), _require(r, "experts", int, where),
                    _require(r, "top", int, where), _opt(r, "identity", int, where) or 0,
                    0 if shared is None else _require(_obj(shared, "mlp.shared", where), "ff", int, where))
            if (f.experts <= 0 or f.identity < 0 or not (0 < f.top <= f.experts + f.identity)
                    or f.shared < (0 if shared is None else 1)):
                raise ConfigError(f"{where}: {f.top} of {f.experts} + {f.identity} experts (shared: {f.shared}) cannot be run")
        else:
            raise ConfigError(f"{where}: unknown mlp kind {kind!r} (dense, moe)")
        if f.ff <= 0:
            raise ConfigError(f"{where}: the feed-forward's inner size must be positive")
        return f

    def to_dict(self) -> Dict[str, Any]:
        if self.kind == "dense":
            return {"kind": "dense", "ff": self.ff}
        router = {"experts": self.experts, "top": self.top}
        if self.identity:
            router["identity"] = self.identity
        out: Dict[str, Any] = {"kind": "moe", "expert": {"ff": self.ff}, "router": router}
        if self.shared:
            out["shared"] = {"ff": self.shared}
        return out

    def spec(self, cfg: "LitizenConfig") -> PartSpec:
        if self.kind == "dense":
            return PartSpec("gated_mlp", dict(hidden_size=cfg.width, intermediate_size=self.ff, activation="silu",
                                              names={"gate": "gate", "up": "up", "down": "down"}))
        params: Dict[str, Any] = dict(
            hidden_size=cfg.width, intermediate_size=self.ff, num_experts=self.experts, top=self.top, identity=self.identity,
            activation="silu", scores="all", correction=True,
            names={"router": "router", "correction": "correction", "gate": "e{i}.gate", "up": "e{i}.up", "down": "e{i}.down",
                   "shared_gate": "shared.gate", "shared_up": "shared.up", "shared_down": "shared.down"})
        if self.shared:
            params["shared"] = dict(intermediate_size=self.shared)
        return PartSpec("routed_experts", params)


@dataclass(frozen=True)
class LitizenLayer:
    type: str
    mixer: Any
    ff: Optional[FeedForward]          # None: no feed-forward


@dataclass(frozen=True)
class LitizenConfig:
    vocab: int
    width: int
    norm_eps: float
    layers: Tuple[LitizenLayer, ...]
    norm_groups: int = 1
    taps: int = 0                      # canon.taps; 0: nothing in front of the mixers
    embedding_scale: float = 1.0
    logit_softcap: Optional[float] = None
    max_positions: int = DEFAULT_POSITIONS
    eos_token_id: Optional[Tuple[int, ...]] = None
    architecture: str = "Litizen"

    @classmethod
    def from_dict(cls, raw: Dict[str, Any], where: str = "config.json") -> "LitizenConfig":
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError(f"{where}: 'layers' must be a list of layers")
        out = []
        for i, l in enumerate(layers):
            at = f"{where}: layers[{i}]"
            l = _obj(l, f"layers[{i}]", where)
            kind = _require(l, "type", str, at)
            if kind not in MIXERS:
                raise ConfigError(f"{at}: unknown layer type {kind!r} ({', '.join(MIXERS)})")
            out.append(LitizenLayer(kind, MIXERS[kind].from_dict(l.get("mixer"), at),
                                    None if l.get("mlp") is None else FeedForward.from_dict(l["mlp"], at)))
        norm = _obj(raw.get("norm"), "norm", where)
        canon, emb, eos = raw.get("canon"), raw.get("embedding"), raw.get("eos_token_id")
        scale = None if emb is None else _opt(_obj(emb, "embedding", where), "scale", float, where)
        cfg = cls(vocab=_require(raw, "vocab", int, where), width=_require(raw, "width", int, where),
                  norm_eps=_require(norm, "eps", float, where), layers=tuple(out), norm_groups=_opt(norm, "groups", int, where) or 1,
                  taps=0 if canon is None else _require(_obj(canon, "canon", where), "taps", int, where),
                  embedding_scale=1.0 if scale is None else scale,
                  logit_softcap=_opt(raw, "logit_softcap", float, where),
                  max_positions=_opt(raw, "max_positions", int, where) or DEFAULT_POSITIONS,
                  eos_token_id=None if eos is None else tuple(int(e) for e in (eos if isinstance(eos, list) else [eos])),
                  architecture=str(raw.get("architecture") or (raw.get("architectures") or ["Litizen"])[0]))
        if min(cfg.vocab, cfg.width, cfg.max_positions, cfg.norm_groups) <= 0 or cfg.width % cfg.norm_groups:
            raise ConfigError(f"{where}: vocab, width and max_positions must be positive, and norm.groups divide the width")
        if cfg.taps < (0 if canon is None else 1) or (cfg.logit_softcap is not None and not cfg.logit_softcap > 0):
            raise ConfigError(f"{where}: canon.taps and logit_softcap must be positive or absent")
        return cfg

    def to_dict(self) -> Dict[str, Any]:
        layers = [{"type": l.type, "mixer": l.mixer.to_dict(), "mlp": None if l.ff is None else l.ff.to_dict()} for l in self.layers]
        out: Dict[str, Any] = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
                               "norm": {"eps": self.norm_eps, "groups": self.norm_groups},
                               "embedding": {"scale": self.embedding_scale}, "layers": layers}
        if self.taps:
            out["canon"] = {"taps": self.taps}
        if self.logit_softcap is not None:
            out["logit_softcap"] = self.logit_softcap
        if self.max_positions != DEFAULT_POSITIONS:
            out["max_positions"] = self.max_positions
        if self.eos_token_id is not None:
            out["eos_token_id"] = list(self.eos_token_id)
        return out


def litizen_spec(cfg: LitizenConfig) -> ModelSpec:
    def norm(name: str) -> PartSpec:
        return PartSpec("rmsnorm", dict(dim=cfg.width, eps=cfg.norm_eps, name=name, groups=cfg.norm_groups))

    layers = []
    for i, l in enumerate(cfg.layers):
        mixer = l.mixer.spec(cfg)
        if cfg.taps:
            mixer = PartSpec("input_conv", dict(hidden_size=cfg.width, taps=cfg.taps, name=f"l{i}.canon1", inner=mixer))
        names = ("norm1", "norm1b") + (("norm2", "norm2b") if l.ff is not None else ())
        layers.append(LayerSpec(prefix=f"l{i}", block="sandwich", mixer=mixer, feed_forward=None if l.ff is None else l.ff.spec(cfg),
                                norms={n: norm(f"l{i}.{n}") for n in names}, mixer_name="mix", feed_forward_name="mlp"))
    return ModelSpec(
        architecture=cfg.architecture, vocab_size=cfg.vocab, hidden_size=cfg.width, max_positions=cfg.max_positions,
        embedding=PartSpec("embedding", dict(name="embed", vocab_size=cfg.vocab, dim=cfg.width, scale=cfg.embedding_scale)),
        layers=tuple(layers), schedule=tuple(ScheduleEntry(i) for i in range(len(layers))), final_norm=norm("final.norm"),
        head=PartSpec("lm_head", dict(name="head", tied=False, vocab_size=cfg.vocab, dim=cfg.width, softcap=cfg.logit_softcap)),
        eos_token_ids=tuple(cfg.eos_token_id or ()))


LITIZEN = ModelFamily("litizen", LitizenConfig, litizen_spec)
register_architecture("Litizen", LITIZEN)
