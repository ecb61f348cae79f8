"""Tisosun as data: its config.json typed, and turned into a `ModelSpec`.

A decoder-only model whose layers are listed one by one in config.json (`layers`: each entry a `type`, the mixer's sizes
under `mixer`, and `mlp` or null).  What the design fixes is written here; what config.json gives is read from there:

  embedding   X_0 = N(embed[token]); every model norm (the embedding's, the layers', the last one) is N(x) = x * rsqrt(mean(x^2)
              + eps) * (1 + w): the tensor holds the factor's distance from one
  layer i     x' = x + mixer(norm1(x)) + ff(norm2(x)), both branches of the same x (block "parallel"; `mlp: null` leaves the
              second out); X_(i+1) = x' plus the layer's own input for the token (stream op "token_side", `token_side.dim`
              columns a layer of the table `side.embed`); what the next layer gets is sum_(j <= i+1) dwa[j] X_j (stream op
              "depth_average")
  type "mingru"    a gated recurrence of one number a channel whose gates read the current token alone (`parts/channel.py`)
  type "rglru"     Griffin's recurrent block: a short convolution and a real-gated linear recurrent unit (`parts/channel.py`)
  type "parallel"  two mixers on the same input, each RMS-normed over the width with a weight of its own, half their sum:
              left   grouped-query softmax attention within chunks of mask.size positions, biases on q, k and v, q and k
                     RMS-normed head by head with a weight, rotary positions on the first rot.dims dims in pairs (2i, 2i + 1)
                     (rot.scaling: frequencies blended along a ramp), score softcap * tanh((q . k) scale / softcap), value
                     heads of their own size
              right  lightning attention (`parts/recurrent.py`): silu on q, k and v, one constant decay a head, the heads
                     normed together, times sigmoid(g h)
  mlp         dense: down(silu(gate h) * (up h))
  output      the norm `final.norm`, `head`

Tensor names: `embed`, `embed.norm`, `side.embed`, `l<i>.norm1`, `l<i>.norm2`, `l<i>.mix.*` (in "parallel" `l<i>.mix.left.*`,
`l<i>.mix.right.*`, with the branches' norms `.left.out` and `.right.out`), `l<i>.mlp.{gate,up,down}`, `l<i>.side.{gate,proj,norm}`,
`l<i>.dwa`, `final.norm`, `head`.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from ..config.model_config import ConfigError, _require, _typed
from ..config.spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry
from .debusun import Rotary, _window
from .lilalorn import RetentionBranch
from .registry import ModelFamily, register_architecture

DEFAULT_POSITIONS = 1 << 15       # config.json names no longest sequence: what the engine plans its tables for
BRANCH_SCALE = 0.5                # of each of the two mixers side by side


def _obj(raw: Any, what: str, where: str) -> Dict[str, Any]:
    if not isinstance(raw, dict):
        raise ConfigError(f"{where}: {what!r} must be an object")
    return raw


def _opt(raw: Optional[Dict[str, Any]], key: str, typ, where: str):
    return None if not raw or raw.get(key) is None else _typed(raw[key], key, typ, where)


@dataclass(frozen=True)
class MinGruMixer:
    width: int

    @classmethod
    def from_dict(cls, raw: Any, where: str) -> "MinGruMixer":
        m = cls(_require(_obj(raw, "mixer", where), "width", int, where))
        if m.width <= 0:
            raise ConfigError(f"{where}: a recurrence of {m.width} channels cannot be run")
        return m

    def to_dict(self) -> Dict[str, Any]:
        return {"width": self.width}

    def spec(self, cfg: "TisosunConfig") -> PartSpec:
        return PartSpec("mingru", dict(hidden_size=cfg.width, width=self.width))


@dataclass(frozen=True)
class RgLruMixer:
    width: int
    blocks: int
    conv: int

    @classmethod
    def from_dict(cls, raw: Any, where: str) -> "RgLruMixer":
        raw = _obj(raw, "mixer", where)
        m = cls(*(_require(raw, k, int, where) for k in ("width", "blocks", "conv")))
        if min(m.width, m.blocks, m.conv) <= 0 or m.width % m.blocks:
            raise ConfigError(f"{where}: {m.width} channels in {m.blocks} blocks behind {m.conv} taps cannot be run")
        return m

    def to_dict(self) -> Dict[str, Any]:
        return {"width": self.width, "blocks": self.blocks, "conv": self.conv}

    def spec(self, cfg: "TisosunConfig") -> PartSpec:
        return PartSpec("rglru", dict(hidden_size=cfg.width, width=self.width, blocks=self.blocks, conv=self.conv))


@dataclass(frozen=True)
class ChunkedBranch:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: Optional[float]
    chunk: int                         # mask.size; 0: every earlier token is seen
    rot: Optional[Rotary]

    @classmethod
    def from_dict(cls, raw: Any, where: str) -> "ChunkedBranch":
        raw = _obj(raw, "left", where)
        dim = _require(raw, "dim", int, where)
        b = cls(_require(raw, "heads", int, where), _require(raw, "kv_heads", int, where), dim, _opt(raw, "vdim", int, where) or dim,
                _require(raw, "scale", float, where), _opt(raw, "softcap", float, where), _window(raw, where),
                Rotary.from_dict(raw["rot"], where) if raw.get("rot") is not None else None)
        if min(b.heads, b.kv_heads, b.dim, b.vdim) <= 0 or b.heads % b.kv_heads:
            raise ConfigError(f"{where}: {b.heads} heads of {b.dim}/{b.vdim} on {b.kv_heads} kv heads cannot be run")
        if b.softcap is not None and not b.softcap > 0:
            raise ConfigError(f"{where}: softcap must be positive or absent")
        if b.rot is not None and b.rot.dims > b.dim:
            raise ConfigError(f"{where}: {b.rot.dims} rotated dims of a head of {b.dim}")
        return b

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.softcap is not None:
            out["softcap"] = self.softcap
        if self.chunk:
            out["mask"] = {"size": self.chunk}
        if self.rot is not None:
            out["rot"] = self.rot.to_dict()
        return out

    def spec(self, cfg: "TisosunConfig") -> PartSpec:
        position = None
        if self.rot is not None:
            rope = self.rot.spec(self.dim, cfg.max_positions)
            position = PartSpec(rope.kind, dict(rope.params, precise=True))
        return PartSpec("attention", dict(
            hidden_size=cfg.width, num_heads=self.heads, num_kv_heads=self.kv_heads, head_dim=self.dim, value_dim=self.vdim, bias=True,
            qk_norm=True, qk_norm_eps=cfg.norm_eps, window=None, chunk=self.chunk, scale=self.scale, score_softcap=self.softcap,
            position=position, general=True,
            names={"q": "q", "k": "k", "v": "v", "o": "o", "q_bias": "q.b", "k_bias": "k.b", "v_bias": "v.b", "q_norm": "q.norm",
                   "k_norm": "k.norm"}))


@dataclass(frozen=True)
class ParallelMixer:
    left: ChunkedBranch
    right: RetentionBranch

    @classmethod
    def from_dict(cls, raw: Any, where: str) -> "ParallelMixer":
        raw = _obj(raw, "mixer", where)
        return cls(ChunkedBranch.from_dict(raw.get("left"), where), RetentionBranch.from_dict(raw.get("right"), where))

    def to_dict(self) -> Dict[str, Any]:
        return {"left": self.left.to_dict(), "right": self.right.to_dict()}

    def spec(self, cfg: "TisosunConfig") -> PartSpec:
        r = self.right
        right = PartSpec("lightning_attention", dict(hidden_size=cfg.width, num_heads=r.heads, key_dim=r.dim, value_dim=r.vdim,
                                                     decay=r.decay, norm_eps=cfg.norm_eps))
        return PartSpec("parallel", dict(hidden_size=cfg.width, out_norm=cfg.norm_eps, out_norm_name="out",
                                         branches=(("left", BRANCH_SCALE, self.left.spec(cfg)), ("right", BRANCH_SCALE, right))))


MIXERS = {"mingru": MinGruMixer, "parallel": ParallelMixer, "rglru": RgLruMixer}


@dataclass(frozen=True)
class TisosunLayer:
    type: str
    mixer: Any
    ff: Optional[int]                  # inner size of the dense feed-forward; None: no feed-forward


@dataclass(frozen=True)
class TisosunConfig:
    vocab: int
    width: int
    norm_eps: float
    layers: Tuple[TisosunLayer, ...]
    side_dim: int = 0                  # token_side.dim; 0: the layers have no input of their own for the token
    max_positions: int = DEFAULT_POSITIONS
    eos_token_id: Optional[Tuple[int, ...]] = None
    architecture: str = "Tisosun"

    @classmethod
    def from_dict(cls, raw: Dict[str, Any], where: str = "config.json") -> "TisosunConfig":
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
            ff = None
            if l.get("mlp") is not None:
                mlp = _obj(l["mlp"], "mlp", at)
                if str(mlp.get("kind", "dense")) != "dense":
                    raise ConfigError(f"{at}: unknown mlp kind {mlp.get('kind')!r} (dense)")
                ff = _require(mlp, "ff", int, at)
                if ff <= 0:
                    raise ConfigError(f"{at}: the feed-forward's inner size must be positive")
            out.append(TisosunLayer(kind, MIXERS[kind].from_dict(l.get("mixer"), at), ff))
        side = raw.get("token_side")
        eos = raw.get("eos_token_id")
        cfg = cls(vocab=_require(raw, "vocab", int, where), width=_require(raw, "width", int, where),
                  norm_eps=_require(_obj(raw.get("norm"), "norm", where), "eps", float, where), layers=tuple(out),
                  side_dim=0 if side is None else _require(_obj(side, "token_side", where), "dim", int, where),
                  max_positions=_opt(raw, "max_positions", int, where) or DEFAULT_POSITIONS,
                  eos_token_id=None if eos is None else tuple(int(e) for e in (eos if isinstance(eos, list) else [eos])),
                  architecture=str(raw.get("architecture") or (raw.get("architectures") or ["Tisosun"])[0]))
        if cfg.vocab <= 0 or cfg.width <= 0 or cfg.max_positions <= 0 or cfg.side_dim < (1 if side is not None else 0):
            raise ConfigError(f"{where}: vocab, width, max_positions and token_side.dim must be positive")
        return cfg

    def to_dict(self) -> Dict[str, Any]:
        layers = [{"type": l.type, "mixer": l.mixer.to_dict(), "mlp": None if l.ff is None else {"kind": "dense", "ff": l.ff}}
                  for l in self.layers]
        out: Dict[str, Any] = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
                               "norm": {"eps": self.norm_eps}, "layers": layers}
        if self.side_dim:
            out["token_side"] = {"dim": self.side_dim}
        if self.max_positions != DEFAULT_POSITIONS:
            out["max_positions"] = self.max_positions
        if self.eos_token_id is not None:
            out["eos_token_id"] = list(self.eos_token_id)
        return out


def tisosun_spec(cfg: TisosunConfig) -> ModelSpec:
    n = len(cfg.layers)

    def norm(name: str) -> PartSpec:
        return PartSpec("rmsnorm", dict(dim=cfg.width, eps=cfg.norm_eps, name=name, weight_offset=1.0))

    layers, schedule = [], []
    for i, l in enumerate(cfg.layers):
        norms = {"norm1": norm(f"l{i}.norm1")}
        ffn = None
        if l.ff is not None:
            norms["norm2"] = norm(f"l{i}.norm2")
            ffn = PartSpec("gated_mlp", dict(hidden_size=cfg.width, intermediate_size=l.ff, activation="silu",
                                             names={"gate": "gate", "up": "up", "down": "down"}))
        layers.append(LayerSpec(prefix=f"l{i}", block="parallel", mixer=l.mixer.spec(cfg), feed_forward=ffn, norms=norms,
                                mixer_name="mix", feed_forward_name="mlp"))
        after = []
        if cfg.side_dim:
            after.append(PartSpec("token_side", dict(hidden_size=cfg.width, vocab_size=cfg.vocab, dim=cfg.side_dim,
                                                     offset=i * cfg.side_dim, row=n * cfg.side_dim, table="side.embed",
                                                     prefix=f"l{i}.side", norm_eps=cfg.norm_eps)))
        after.append(PartSpec("depth_average", dict(name=f"l{i}.dwa", place=i, layers=n)))
        schedule.append(ScheduleEntry(i, after=tuple(after)))
    return ModelSpec(
        architecture=cfg.architecture, vocab_size=cfg.vocab, hidden_size=cfg.width, max_positions=cfg.max_positions,
        embedding=PartSpec("embedding", dict(name="embed", vocab_size=cfg.vocab, dim=cfg.width,
                                             norm=dict(name="embed.norm", eps=cfg.norm_eps, weight_offset=1.0))),
        layers=tuple(layers), schedule=tuple(schedule), final_norm=norm("final.norm"),
        head=PartSpec("lm_head", dict(name="head", tied=False, vocab_size=cfg.vocab, dim=cfg.width)),
        eos_token_ids=tuple(cfg.eos_token_id or ()))


TISOSUN = ModelFamily("tisosun", TisosunConfig, tisosun_spec)
register_architecture("Tisosun", TISOSUN)
