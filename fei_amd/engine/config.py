"""Model specs for the local engine.

Three families of decoder: ``ModelSpec`` (one attention layer repeated;
Llama-3), ``TobaraxSpec`` (a list of unlike layers, each with its own mixer
and sizes, part of the list run several times in a row) and ``BokenexSpec`` (a
list of parallel layers: sigmoid attention beside a dense feed-forward or a
mixture of experts). ``get_spec`` takes a registered name or a folder with a
config.json.

Llama-3 8B/70B shapes per the BASELINE.json configs (weights are random-init
— there is no network for checkpoints; bench.py states data=synthetic).
``llama3-tiny`` exists for CPU tests; ``bge-base`` shapes the memdir
embedding encoder (fei_amd/models/bge.py).
"""

from __future__ import annotations

import json
import os
import struct
from dataclasses import dataclass, fields
from typing import Any, Dict, List, Optional, Tuple, Union


@dataclass(frozen=True)
class ModelSpec:
    name: str
    vocab_size: int
    hidden_size: int
    num_layers: int
    num_heads: int
    num_kv_heads: int
    head_dim: int
    intermediate_size: int
    rope_theta: float = 500000.0
    norm_eps: float = 1e-5
    max_seq_len: int = 8192
    arch: str = "llama"           # "llama" (decoder) | "bert" (encoder)

    max_positions = None          # positions past which it cannot go

    @property
    def q_size(self) -> int:
        return self.num_heads * self.head_dim

    @property
    def kv_size(self) -> int:
        return self.num_kv_heads * self.head_dim

    def params_bytes(self, dtype_bytes: int = 2) -> int:
        """Approximate parameter bytes (embeddings + blocks + head)."""
        h, i, v = self.hidden_size, self.intermediate_size, self.vocab_size
        per_layer = (h * (self.q_size + 2 * self.kv_size)   # qkv
                     + self.q_size * h                      # o
                     + 3 * h * i                            # gate/up/down
                     + 2 * h)                               # norms
        total = v * h * 2 + self.num_layers * per_layer + h
        return total * dtype_bytes


# -- decoders made of unlike layers -------------------------------------------

@dataclass(frozen=True)
class LatentAttentionSpec:
    """Attention whose keys and values are linear maps of a cached latent.

    Per head ``dim`` unrotated and ``rot_dim`` rotated query/key dimensions
    and ``vdim`` value dimensions; the rotated key part is shared by the
    heads. ``window``: a query sees that many positions, itself included
    (None = all)."""
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot_base: float
    window: Optional[int] = None

    kind = "latent_attention"

    @property
    def in_rows(self) -> int:
        """Output rows of the stacked projections of the mixer's input."""
        return (self.heads * (self.dim + self.rot_dim) + self.kv_rank +
                self.rot_dim + self.heads * self.vdim)

    @property
    def out_cols(self) -> int:
        return self.heads * self.vdim

    @property
    def row_width(self) -> int:
        """Cached values per token."""
        return self.kv_rank + self.rot_dim


@dataclass(frozen=True)
class GLASpec:
    """Gated linear attention: a [dim, vdim] state per head, decayed per key
    channel by sigmoid(z)^(1/tau), z a rank-``gate_rank`` map of the input."""
    heads: int
    dim: int
    vdim: int
    tau: float
    gate_rank: int

    kind = "gla"

    @property
    def in_rows(self) -> int:
        return (2 * self.heads * self.dim + 2 * self.heads * self.vdim +
                self.gate_rank)

    @property
    def out_cols(self) -> int:
        return self.heads * self.vdim

    @property
    def state_size(self) -> int:
        """State values per sequence."""
        return self.heads * self.dim * self.vdim


@dataclass(frozen=True)
class SigmoidAttentionSpec:
    """Grouped-query attention whose key weights are sigmoids, not a softmax.

    q, k and v pass a causal convolution of ``conv`` taps per channel; q and k
    an RMS norm per head. A score is scale * (q . k) - r1 ln(1 + r2 d) at
    distance d, a weight sigmoid(score + pb), with r1, r2, pb per head.
    ``window``: a query sees that many positions, itself included (None =
    all)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    conv: int = 1
    window: Optional[int] = None

    kind = "attention"

    @property
    def in_rows(self) -> int:
        """Rows of the stacked q, k, v projections."""
        return self.heads * self.dim + self.row_width

    @property
    def out_cols(self) -> int:
        return self.heads * self.vdim

    @property
    def row_width(self) -> int:
        """Cached values per token: keys, then values, of every kv head."""
        return self.kv_heads * (self.dim + self.vdim)


MixerSpec = Union[LatentAttentionSpec, GLASpec, SigmoidAttentionSpec]


@dataclass(frozen=True)
class DenseSpec:
    """W_down relu(W_up h)^2."""
    ff: int

    kind = "dense"


@dataclass(frozen=True)
class MoESpec:
    """``top`` of ``experts`` feed-forwards of width ``ff`` per token, by
    sigmoid router scores; their weights are the chosen scores over their sum,
    times ``scale``."""
    experts: int
    top: int
    ff: int
    scale: float = 1.0

    kind = "moe"


MlpSpec = Union[DenseSpec, MoESpec]


@dataclass(frozen=True)
class LayerSpec:
    mixer: MixerSpec
    ff: Optional[int] = None          # width of the feed-forward; None = none


@dataclass(frozen=True)
class LoopSpec:
    """Layers start .. stop-1 run ``times`` times with the same weights."""
    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class LayerRun:
    layer: int                        # index into the weights
    enters_pass: Optional[int] = None  # number of the pass that starts here


def _only(d: Dict[str, Any], allowed, where: str) -> None:
    extra = sorted(set(d) - set(allowed))
    if extra:
        raise ValueError(f"unknown keys {extra} in {where}")


@dataclass(frozen=True)
class TobaraxSpec:
    name: str
    vocab_size: int
    hidden_size: int
    layers: Tuple[LayerSpec, ...]
    norm_eps: float
    logit_scale: float
    logit_softcap: Optional[float] = None
    loop: Optional[LoopSpec] = None
    max_seq_len: int = 8192
    arch: str = "tobarax"

    max_positions = None          # rotations have no last position

    def __post_init__(self) -> None:
        if self.loop is not None:
            lp = self.loop
            if not (0 <= lp.start < lp.stop <= len(self.layers)
                    and lp.times >= 1):
                raise ValueError(f"loop {lp} does not fit "
                                 f"{len(self.layers)} layers")
        for L in self.layers:
            if L.mixer.kind == "latent_attention" and L.mixer.rot_dim % 2:
                raise ValueError("rotated dimensions come in pairs")

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    @property
    def intermediate_size(self) -> int:
        """Widest feed-forward."""
        return max((L.ff or 0 for L in self.layers), default=0)

    @property
    def runs(self) -> Tuple[LayerRun, ...]:
        """Layer runs in execution order; each has its own cache or state."""
        n, lp = len(self.layers), self.loop
        if lp is None:
            return tuple(LayerRun(i) for i in range(n))
        out: List[LayerRun] = [LayerRun(i) for i in range(lp.start)]
        for t in range(lp.times):
            out += [LayerRun(i, t if i == lp.start else None)
                    for i in range(lp.start, lp.stop)]
        return tuple(out + [LayerRun(i) for i in range(lp.stop, n)])

    def params_bytes(self, dtype_bytes: int = 2) -> int:
        C = self.hidden_size
        total = 2 * self.vocab_size * C + C
        for L in self.layers:
            m = L.mixer
            total += C * m.in_rows + C * m.out_cols + C
            if m.kind == "latent_attention":
                total += m.kv_rank * (1 + m.heads * (m.dim + m.vdim))
            else:
                total += m.vdim + m.heads * m.dim * (m.gate_rank + 1)
            if L.ff:
                total += 3 * C * L.ff + C
        if self.loop is not None:
            total += 2 * C * C + self.loop.times * C
        return total * dtype_bytes

    # -- config.json -----------------------------------------------------------

    @classmethod
    def from_config(cls, cfg: Dict[str, Any], shapes: Dict[str, Tuple[int, ...]],
                    name: str = "tobarax",
                    max_seq_len: int = 8192) -> "TobaraxSpec":
        """``shapes`` gives the sizes that only the tensors have (the rank of
        a decay gate). Keys that this class does not know are refused rather
        than skipped."""
        _only(cfg, ("architecture", "layers", "logit_scale", "logit_softcap",
                    "loop", "norm", "vocab", "width", "max_seq_len"), "config")
        layers = []
        for i, L in enumerate(cfg["layers"]):
            where = f"layer {i}"
            _only(L, ("type", "mixer", "mlp"), where)
            m, mlp = L["mixer"], L.get("mlp")
            if L["type"] == "latent_attention":
                _only(m, ("heads", "dim", "rot_dim", "vdim", "kv_rank",
                          "scale", "rot", "mask"), where)
                rot, mask = m.get("rot") or {}, m.get("mask") or {}
                _only(rot, ("base", "dims"), where)
                _only(mask, ("size",), where)
                if rot.get("dims", m["rot_dim"]) != m["rot_dim"]:
                    raise ValueError(f"{where}: the whole rotated part is "
                                     "rotated, rot.dims must be rot_dim")
                mixer: MixerSpec = LatentAttentionSpec(
                    heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"],
                    vdim=m["vdim"], kv_rank=m["kv_rank"],
                    scale=float(m["scale"]),
                    rot_base=float(rot.get("base", 10000.0)),
                    window=mask.get("size"))
            elif L["type"] == "gla":
                _only(m, ("heads", "dim", "vdim", "tau"), where)
                mixer = GLASpec(
                    heads=m["heads"], dim=m["dim"], vdim=m["vdim"],
                    tau=float(m["tau"]),
                    gate_rank=int(shapes[f"l{i}.mix.a1"][0]))
            else:
                raise ValueError(f"{where}: unknown type {L['type']!r}")
            ff = None
            if mlp is not None:
                _only(mlp, ("kind", "ff"), where)
                if mlp.get("kind", "dense") != "dense":
                    raise ValueError(f"{where}: unknown mlp {mlp['kind']!r}")
                ff = int(mlp["ff"])
            layers.append(LayerSpec(mixer, ff))
        loop = cfg.get("loop")
        return cls(
            name=name, vocab_size=cfg["vocab"], hidden_size=cfg["width"],
            layers=tuple(layers), norm_eps=float(cfg["norm"]["eps"]),
            logit_scale=float(cfg.get("logit_scale", 1.0)),
            logit_softcap=cfg.get("logit_softcap"),
            loop=LoopSpec(**loop) if loop else None,
            max_seq_len=int(cfg.get("max_seq_len", max_seq_len)))

    def to_config(self) -> Dict[str, Any]:
        layers = []
        for L in self.layers:
            m = L.mixer
            if m.kind == "latent_attention":
                mixer = {"heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim,
                         "vdim": m.vdim, "kv_rank": m.kv_rank,
                         "scale": m.scale,
                         "rot": {"base": m.rot_base, "dims": m.rot_dim}}
                if m.window is not None:
                    mixer["mask"] = {"size": m.window}
            else:
                mixer = {"heads": m.heads, "dim": m.dim, "vdim": m.vdim,
                         "tau": m.tau}
            layers.append({"type": m.kind, "mixer": mixer,
                           "mlp": None if L.ff is None else
                           {"kind": "dense", "ff": L.ff}})
        out = {"architecture": "Tobarax", "layers": layers,
               "logit_scale": self.logit_scale,
               "logit_softcap": self.logit_softcap,
               "norm": {"eps": self.norm_eps}, "vocab": self.vocab_size,
               "width": self.hidden_size, "max_seq_len": self.max_seq_len}
        if self.loop is not None:
            out["loop"] = {"start": self.loop.start, "stop": self.loop.stop,
                           "times": self.loop.times}
        return out


@dataclass(frozen=True)
class ParallelLayerSpec:
    """Mixer and feed-forward read the same normed input."""
    mixer: SigmoidAttentionSpec
    mlp: Optional[MlpSpec] = None


@dataclass(frozen=True)
class BokenexSpec:
    """``max_seq_len`` is the number of learned position vectors."""
    name: str
    vocab_size: int
    hidden_size: int
    layers: Tuple[ParallelLayerSpec, ...]
    norm_eps: float
    residual_mult: float
    max_seq_len: int
    arch: str = "bokenex"

    @property
    def max_positions(self) -> Optional[int]:
        """Positions past which the model cannot go."""
        return self.max_seq_len

    def __post_init__(self) -> None:
        for i, L in enumerate(self.layers):
            m = L.mixer
            if min(m.heads, m.kv_heads, m.dim, m.vdim, m.conv) < 1 \
                    or m.heads % m.kv_heads \
                    or (m.window is not None and m.window < 1):
                raise ValueError(f"layer {i}: impossible mixer {m}")
            if L.mlp is not None and L.mlp.kind == "moe" and \
                    not 1 <= L.mlp.top <= L.mlp.experts:
                raise ValueError(f"layer {i}: {L.mlp.top} of "
                                 f"{L.mlp.experts} experts")

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    @property
    def intermediate_size(self) -> int:
        """Widest feed-forward, all experts of a layer together."""
        return max((L.mlp.ff * getattr(L.mlp, "experts", 1)
                    for L in self.layers if L.mlp is not None), default=0)

    def params_bytes(self, dtype_bytes: int = 2) -> int:
        C = self.hidden_size
        total = (2 * self.vocab_size + self.max_seq_len) * C + 1
        for L in self.layers:
            m = L.mixer
            total += (C + m.conv) * m.in_rows + C * m.out_cols
            total += 2 * m.dim + 3 * m.heads + 1
            if L.mlp is not None and L.mlp.kind == "moe":
                total += L.mlp.experts * C * (1 + 2 * L.mlp.ff)
            elif L.mlp is not None:
                total += 2 * C * L.mlp.ff
        return total * dtype_bytes

    # -- config.json -----------------------------------------------------------

    @classmethod
    def from_config(cls, cfg: Dict[str, Any], shapes: Dict[str, Tuple[int, ...]],
                    name: str = "bokenex") -> "BokenexSpec":
        """Keys that this class does not know are refused rather than
        skipped. ``shapes`` is not needed: the configuration has all sizes."""
        _only(cfg, ("architecture", "layers", "max_positions", "norm",
                    "residual_mult", "vocab", "width"), "config")
        layers = []
        for i, L in enumerate(cfg["layers"]):
            where = f"layer {i}"
            _only(L, ("type", "mixer", "mlp"), where)
            if L["type"] != "attention":
                raise ValueError(f"{where}: unknown type {L['type']!r}")
            m, mask = L["mixer"], L["mixer"].get("mask") or {}
            _only(m, ("conv", "dim", "heads", "kv_heads", "mask", "scale",
                      "vdim"), where)
            _only(mask, ("size",), where)
            mixer = SigmoidAttentionSpec(
                heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
                vdim=m["vdim"], scale=float(m["scale"]), conv=m["conv"],
                window=mask.get("size"))
            layers.append(ParallelLayerSpec(
                mixer, _mlp(L["mlp"], where) if L.get("mlp") else None))
        return cls(
            name=name, vocab_size=cfg["vocab"], hidden_size=cfg["width"],
            layers=tuple(layers), norm_eps=float(cfg["norm"]["eps"]),
            residual_mult=float(cfg["residual_mult"]),
            max_seq_len=int(cfg["max_positions"]))

    def to_config(self) -> Dict[str, Any]:
        layers = []
        for L in self.layers:
            m, f = L.mixer, L.mlp
            mixer = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim,
                     "vdim": m.vdim, "scale": m.scale, "conv": m.conv}
            if m.window is not None:
                mixer["mask"] = {"size": m.window}
            mlp = None
            if f is not None and f.kind == "moe":
                mlp = {"kind": "moe", "expert": {"ff": f.ff},
                       "router": {"experts": f.experts, "top": f.top,
                                  "scale": f.scale}}
            elif f is not None:
                mlp = {"kind": "dense", "ff": f.ff}
            layers.append({"type": m.kind, "mixer": mixer, "mlp": mlp})
        return {"architecture": "Bokenex", "layers": layers,
                "max_positions": self.max_seq_len,
                "norm": {"eps": self.norm_eps},
                "residual_mult": self.residual_mult,
                "vocab": self.vocab_size, "width": self.hidden_size}


def _mlp(f: Dict[str, Any], where: str) -> MlpSpec:
    if f["kind"] == "dense":
        _only(f, ("kind", "ff"), where)
        return DenseSpec(int(f["ff"]))
    if f["kind"] != "moe":
        raise ValueError(f"{where}: unknown mlp {f['kind']!r}")
    r = f["router"]
    _only(f, ("kind", "expert", "router"), where)
    _only(f["expert"], ("ff",), where)
    _only(r, ("experts", "top", "scale"), where)
    return MoESpec(experts=int(r["experts"]), top=int(r["top"]),
                   ff=int(f["expert"]["ff"]), scale=float(r["scale"]))


AnySpec = Union[ModelSpec, TobaraxSpec, BokenexSpec]

# config.json's "architecture" -> spec
ARCHITECTURES = {"Tobarax": TobaraxSpec, "Bokenex": BokenexSpec}


def _tobarax(name: str, vocab: int, width: int, ff: int, heads: int,
             pattern: str, loop: Optional[LoopSpec], dim: int, rot: int,
             vdim: int, kv_rank: int, window: int, gla_heads: int,
             gla_dim: int, gla_vdim: int, gate_rank: int = 16,
             max_seq_len: int = 8192) -> TobaraxSpec:
    """``pattern``: one letter per layer, 'a' latent attention, 'g' GLA."""
    att = LatentAttentionSpec(heads=heads, dim=dim, rot_dim=rot, vdim=vdim,
                              kv_rank=kv_rank, scale=(dim + rot) ** -0.5,
                              rot_base=500000.0, window=window)
    gla = GLASpec(heads=gla_heads, dim=gla_dim, vdim=gla_vdim, tau=16.0,
                  gate_rank=gate_rank)
    return TobaraxSpec(
        name=name, vocab_size=vocab, hidden_size=width,
        layers=tuple(LayerSpec(att if c == "a" else gla, ff) for c in pattern),
        norm_eps=1e-5, logit_scale=0.5, logit_softcap=30.0, loop=loop,
        max_seq_len=max_seq_len)


def _bokenex(name: str, vocab: int, width: int, heads: int, kv_heads: int,
             dim: int, vdim: int, window: int, pattern: str, dense: DenseSpec,
             moe: MoESpec, conv: int = 4,
             max_seq_len: int = 8192) -> BokenexSpec:
    """``pattern``: one letter per layer, 'd' dense, 'm' mixture of experts,
    '-' without a feed-forward."""
    att = SigmoidAttentionSpec(heads=heads, kv_heads=kv_heads, dim=dim,
                               vdim=vdim, scale=dim ** -0.5, conv=conv,
                               window=window)
    mlp = {"d": dense, "m": moe, "-": None}
    return BokenexSpec(
        name=name, vocab_size=vocab, hidden_size=width,
        layers=tuple(ParallelLayerSpec(att, mlp[c]) for c in pattern),
        norm_eps=1e-5, residual_mult=0.5, max_seq_len=max_seq_len)


MODEL_SPECS: Dict[str, AnySpec] = {
    "llama3-8b": ModelSpec(
        name="llama3-8b", vocab_size=128256, hidden_size=4096, num_layers=32,
        num_heads=32, num_kv_heads=8, head_dim=128, intermediate_size=14336,
    ),
    "llama3-70b": ModelSpec(
        name="llama3-70b", vocab_size=128256, hidden_size=8192, num_layers=80,
        num_heads=64, num_kv_heads=8, head_dim=128, intermediate_size=28672,
    ),
    # 1B-ish shape for quick single-GPU smoke/perf probes
    "llama3-1b": ModelSpec(
        name="llama3-1b", vocab_size=128256, hidden_size=2048, num_layers=16,
        num_heads=32, num_kv_heads=8, head_dim=64, intermediate_size=8192,
    ),
    # tiny: CPU tests and GPU numerics tests
    "llama3-tiny": ModelSpec(
        name="llama3-tiny", vocab_size=512, hidden_size=256, num_layers=2,
        num_heads=4, num_kv_heads=2, head_dim=64, intermediate_size=512,
        max_seq_len=512,
    ),
    # tiny8: every sharded axis divisible by 8 — the gloo-8 TP harness
    # (70B's tp=8 shard shape ratios at toy scale)
    "llama3-tiny8": ModelSpec(
        name="llama3-tiny8", vocab_size=512, hidden_size=256, num_layers=2,
        num_heads=8, num_kv_heads=8, head_dim=32, intermediate_size=512,
        max_seq_len=512,
    ),
    # embedding encoder shape (bge-base class): 12L/768h/12heads, D=64
    "bge-base": ModelSpec(
        name="bge-base", vocab_size=30522, hidden_size=768, num_layers=12,
        num_heads=12, num_kv_heads=12, head_dim=64, intermediate_size=3072,
        max_seq_len=512, arch="bert",
    ),
    # Tobarax: latent-attention and GLA layers, a looped block. The 1b/8b
    # shapes have the width, feed-forward and vocabulary of the llama3 specs
    # beside them; tiny is for CPU and numerics tests.
    "tobarax-tiny": _tobarax(
        "tobarax-tiny", vocab=320, width=96, ff=160, heads=3, pattern="agga",
        loop=LoopSpec(1, 3, 2), dim=24, rot=8, vdim=40, kv_rank=56,
        window=48, gla_heads=2, gla_dim=24, gla_vdim=40, gate_rank=8,
        max_seq_len=512),
    "tobarax-1b": _tobarax(
        "tobarax-1b", vocab=128256, width=2048, ff=8192, heads=16,
        pattern="ag" * 7, loop=LoopSpec(6, 8, 2), dim=128, rot=64, vdim=128,
        kv_rank=512, window=1024, gla_heads=8, gla_dim=128, gla_vdim=256),
    "tobarax-8b": _tobarax(
        "tobarax-8b", vocab=128256, width=4096, ff=14336, heads=32,
        pattern="ag" * 15, loop=LoopSpec(14, 16, 2), dim=128, rot=64,
        vdim=128, kv_rank=512, window=4096, gla_heads=16, gla_dim=128,
        gla_vdim=256),
    # Bokenex: layers of sigmoid attention beside a dense feed-forward or a
    # mixture of experts. The 1b/8b shapes have the width, heads and
    # vocabulary of the llama3 specs beside them, and feed-forwards of as many
    # parameters.
    "bokenex-tiny": _bokenex(
        "bokenex-tiny", vocab=304, width=80, heads=4, kv_heads=2, dim=24,
        vdim=40, window=40, pattern="dm-m", dense=DenseSpec(112),
        moe=MoESpec(6, 2, 48, 1.25), conv=3, max_seq_len=512),
    "bokenex-1b": _bokenex(
        "bokenex-1b", vocab=128256, width=2048, heads=32, kv_heads=8, dim=64,
        vdim=64, window=1024, pattern="dm" * 8, dense=DenseSpec(12288),
        moe=MoESpec(16, 4, 768, 1.5)),
    "bokenex-8b": _bokenex(
        "bokenex-8b", vocab=128256, width=4096, heads=32, kv_heads=8, dim=128,
        vdim=128, window=4096, pattern="dm" * 16, dense=DenseSpec(21504),
        moe=MoESpec(16, 4, 1344, 1.5)),
}


def tensor_shapes(path: str) -> Dict[str, Tuple[int, ...]]:
    """Names and shapes in a safetensors file, from its header alone."""
    with open(path, "rb") as f:
        n = struct.unpack("<Q", f.read(8))[0]
        if n > 1 << 28:
            raise ValueError(f"{path}: header of {n} bytes")
        header = json.loads(f.read(n))
    return {k: tuple(v["shape"]) for k, v in header.items()
            if k != "__metadata__"}


def load_spec(path: str) -> AnySpec:
    """Spec of a model folder (config.json + model.safetensors)."""
    with open(os.path.join(path, "config.json"), encoding="utf-8") as f:
        cfg = json.load(f)
    if "arch" in cfg:                      # written by LlamaModel.save_weights
        known = {f.name for f in fields(ModelSpec)}
        return ModelSpec(**{k: v for k, v in cfg.items() if k in known})
    cls = ARCHITECTURES.get(cfg.get("architecture"))
    if cls is None:
        raise ValueError(f"{path}: unknown architecture "
                         f"{cfg.get('architecture')!r}")
    shapes = tensor_shapes(os.path.join(path, "model.safetensors"))
    return cls.from_config(cfg, shapes,
                           name=os.path.basename(os.path.abspath(path)))


def is_model_folder(name: str) -> bool:
    return os.path.isfile(os.path.join(name, "config.json"))


def get_spec(name: str) -> AnySpec:
    """Spec of a registered model, or of a folder with a config.json."""
    if name in MODEL_SPECS:
        return MODEL_SPECS[name]
    if is_model_folder(name):
        return load_spec(name)
    raise KeyError(f"unknown model {name!r}; known: {sorted(MODEL_SPECS)}, "
                   "or a folder with a config.json")
