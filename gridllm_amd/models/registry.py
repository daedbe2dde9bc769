"""Model architecture registry.

The reference has no model definitions at all (compute lived in Ollama);
these specs reproduce the Llama-family architectures its deployments serve
via Ollama model tags (llama3.2:1b, llama3.2:3b,
llama3:70b).
"""

from __future__ import annotations

import json
import os
from dataclasses import dataclass, replace
from typing import Callable, Optional, Union


@dataclass(frozen=True)
class ModelSpec:
    name: str
    hidden: int
    layers: int
    heads: int
    kv_heads: int
    head_dim: int
    intermediate: int
    vocab: int
    rope_theta: float = 500000.0
    norm_eps: float = 1e-5
    max_seq_len: int = 8192
    tie_embeddings: bool = True
    qkv_bias: bool = False         # Qwen2-family: bias on q/k/v projections

    family = "llama"

    def model_info(self) -> dict:
        """Ollama-style model_info of /api/show."""
        return {
            "general.architecture": "llama",
            "general.parameter_count": self.params,
            "llama.block_count": self.layers,
            "llama.embedding_length": self.hidden,
            "llama.attention.head_count": self.heads,
            "llama.attention.head_count_kv": self.kv_heads,
            "llama.feed_forward_length": self.intermediate,
            "llama.context_length": self.max_seq_len,
            "llama.vocab_size": self.vocab,
            "llama.rope.freq_base": self.rope_theta,
        }

    @property
    def params(self) -> int:
        h, f, v = self.hidden, self.intermediate, self.vocab
        qkv = (self.heads + 2 * self.kv_heads) * self.head_dim * h
        o = self.heads * self.head_dim * h
        mlp = 3 * h * f
        if self.qkv_bias:
            qkv += (self.heads + 2 * self.kv_heads) * self.head_dim
        per_layer = qkv + o + mlp + 2 * h
        emb = v * h * (1 if self.tie_embeddings else 2)
        return self.layers * per_layer + emb + h


# ------------------------------------------------------ layer-list designs
# A model whose layers each name a mixer and a feed-forward; a layer may use
# the weights of another one (with a cache or state of its own).


@dataclass(frozen=True)
class AttentionMixer:
    """Grouped softmax attention: unit-RMS q and k, a query temperature
    1 + q_coef ln(floor((p + 1) / q_every) + 1), a sink term and an output
    gate per head; no rotation."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    q_coef: float = 0.0
    q_every: int = 1

    def params(self, width: int) -> int:
        h, g = self.heads, self.kv_heads
        return width * (h * self.dim + g * (self.dim + self.vdim) + h
                        + h * self.vdim) + h


@dataclass(frozen=True)
class MlstmMixer:
    """mLSTM: a matrix memory per head, exponential input gate, log-sigmoid
    forget gate, both soft-capped at gate_cap."""
    heads: int
    dim: int
    vdim: int
    gate_cap: float

    def params(self, width: int) -> int:
        h = self.heads
        return width * h * (2 * self.dim + 3 * self.vdim + 2) \
            + 2 * h + h * self.vdim


@dataclass(frozen=True)
class DenseFF:
    """Gated feed-forward, act(g, u) = g sigmoid(alpha g) (u + shift) with g
    capped at limit and u clamped to +-limit."""
    ff: int
    limit: float
    alpha: float = 1.702
    shift: float = 1.0

    def params(self, width: int) -> int:
        return 3 * width * self.ff


@dataclass(frozen=True)
class RoutedFF:
    """Routed experts with squared ReLU; weights are the softmax over the
    chosen logits."""
    experts: int
    top: int
    ff: int

    def params(self, width: int) -> int:
        return self.experts * width * (2 * self.ff + 1)


@dataclass(frozen=True)
class LayerSpec:
    mixer: Union[AttentionMixer, MlstmMixer]
    ff: Union[DenseFF, RoutedFF, None] = None
    weights_of: Optional[int] = None


@dataclass(frozen=True)
class HybridSpec:
    name: str
    vocab: int
    hidden: int
    layers: tuple[LayerSpec, ...]
    norm_eps: float
    positions: int                 # rows of the learned position table
    max_seq_len: int = 0           # 0 -> positions

    def __post_init__(self) -> None:
        if not 0 < self.max_seq_len <= self.positions:
            object.__setattr__(self, "max_seq_len", self.positions)
        if not self.layers:
            raise ValueError(f"{self.name}: no layers")
        for i, ly in enumerate(self.layers):
            j = self.owner(i)
            own = self.layers[j]
            if (ly.mixer, ly.ff) != (own.mixer, own.ff):
                raise ValueError(f"layer {i} uses layer {j}'s weights but "
                                 "differs from it")
            mx, ff = ly.mixer, ly.ff
            if isinstance(mx, AttentionMixer) and mx.heads % mx.kv_heads:
                raise ValueError(f"layer {i}: {mx.heads} heads over "
                                 f"{mx.kv_heads} key/value heads")
            if isinstance(ff, RoutedFF) and not 0 < ff.top <= ff.experts:
                raise ValueError(f"layer {i}: top {ff.top} of {ff.experts}")

    def owner(self, i: int) -> int:
        """The layer whose tensors layer i uses (itself, usually)."""
        seen = {i}
        while (j := self.layers[i].weights_of) is not None:
            if not 0 <= j < len(self.layers) or j in seen:
                raise ValueError(f"layer {i}: weights_of {j}")
            seen.add(j)
            i = j
        return i

    family = "birepel"

    def model_info(self) -> dict:
        """Ollama-style model_info of /api/show."""
        attn = [ly.mixer for ly in self.layers
                if isinstance(ly.mixer, AttentionMixer)]
        routed = [ly.ff for ly in self.layers if isinstance(ly.ff, RoutedFF)]
        f = self.family
        info = {
            "general.architecture": f,
            "general.parameter_count": self.params,
            f"{f}.block_count": len(self.layers),
            f"{f}.embedding_length": self.hidden,
            f"{f}.context_length": self.max_seq_len,
            f"{f}.vocab_size": self.vocab,
        }
        if attn:
            info |= {f"{f}.attention.block_count": len(attn),
                     f"{f}.attention.head_count": attn[0].heads,
                     f"{f}.attention.head_count_kv": attn[0].kv_heads}
        if routed:
            info |= {f"{f}.expert_count": routed[0].experts,
                     f"{f}.expert_used_count": routed[0].top}
        return info

    @property
    def params(self) -> int:
        w = self.hidden
        total = (self.vocab + self.positions + 1) * w
        for ly in self.layers:
            if ly.weights_of is None:
                total += ly.mixer.params(w) + w
                if ly.ff is not None:
                    total += ly.ff.params(w) + w
        return total


Spec = Union[ModelSpec, HybridSpec]


def _take(d: dict, what: str, keys: tuple, optional: tuple = ()) -> dict:
    """d, if it has all of keys and nothing beyond keys and optional."""
    missing = [k for k in keys if k not in d]
    extra = [k for k in d if k not in keys and k not in optional]
    if missing or extra:
        raise ValueError(f"config: {what} lacks {missing}, has unknown "
                         f"{extra}")
    return d


def _read_mixer(kind: str, d: dict):
    if kind == "attention":
        _take(d, "attention mixer",
              ("heads", "kv_heads", "dim", "vdim", "scale"), ("q_temp",))
        t = d.get("q_temp")
        extra = {}
        if t is not None:
            _take(t, "q_temp", ("coef", "every"))
            extra = {"q_coef": float(t["coef"]), "q_every": int(t["every"])}
        return AttentionMixer(heads=d["heads"], kv_heads=d["kv_heads"],
                              dim=d["dim"], vdim=d["vdim"],
                              scale=float(d["scale"]), **extra)
    if kind == "mlstm":
        _take(d, "mlstm mixer", ("heads", "dim", "vdim", "gate_cap"))
        return MlstmMixer(heads=d["heads"], dim=d["dim"], vdim=d["vdim"],
                          gate_cap=float(d["gate_cap"]))
    raise ValueError(f"config: unknown mixer {kind!r}")


def _read_ff(d: Optional[dict]):
    if d is None:
        return None
    if d.get("kind") == "dense":
        _take(d, "dense mlp", ("kind", "ff", "limit"))
        return DenseFF(ff=d["ff"], limit=float(d["limit"]))
    if d.get("kind") == "moe":
        _take(d, "moe mlp", ("kind", "expert", "router"))
        _take(d["expert"], "expert", ("ff",))
        r = _take(d["router"], "router", ("experts", "top"))
        return RoutedFF(experts=r["experts"], top=r["top"],
                        ff=d["expert"]["ff"])
    raise ValueError(f"config: unknown mlp kind {d.get('kind')!r}")


def read_birepel(cfg: dict, name: str = "birepel") -> HybridSpec:
    """Birepel's config.json -> spec."""
    layers = tuple(
        LayerSpec(mixer=_read_mixer(ly["type"], ly["mixer"]),
                  ff=_read_ff(ly.get("mlp")), weights_of=ly.get("weights_of"))
        for ly in cfg["layers"])
    return HybridSpec(name=name, vocab=cfg["vocab"], hidden=cfg["width"],
                      layers=layers, norm_eps=float(cfg["norm"]["eps"]),
                      positions=cfg["max_positions"])


# "architecture" in config.json -> reader. Checkpoints without that key (HF
# layout) are loaded into the architecture that the model name gives.
_READERS: dict[str, Callable[[dict, str], Spec]] = {"Birepel": read_birepel}


def spec_from_dir(path: str, name: str = "") -> Optional[Spec]:
    """Spec that a checkpoint folder's own config.json gives, under `name`, or
    None if it leaves the architecture to the model name."""
    f = os.path.join(path, "config.json")
    if not path or not os.path.isfile(f):
        return None
    with open(f) as fh:
        cfg = json.load(fh)
    arch = cfg.get("architecture")
    if arch is None:
        return None
    if arch not in _READERS:
        raise ValueError(f"{f}: unknown architecture {arch!r}; known: "
                         f"{sorted(_READERS)}")
    return _READERS[arch](cfg, name or f"{arch.lower()}:custom")


def resolve_spec(model: str, weights_path: str = "",
                 max_seq_len: int = 0) -> Spec:
    """Spec of what an engine is to serve: a checkpoint folder that describes
    itself wins over the name."""
    spec = spec_from_dir(weights_path, model if model not in _SPECS else "")
    if spec is None:
        return get_spec(model, max_seq_len)
    if spec.name not in _SPECS or _SPECS[spec.name] != spec:
        register_spec(spec)
    return replace(spec, max_seq_len=max_seq_len) if max_seq_len else spec


_SPECS: dict[str, Spec] = {}


def _reg(spec: Spec, *aliases: str) -> None:
    _SPECS[spec.name] = spec
    for a in aliases:
        _SPECS[a] = spec


_reg(ModelSpec("llama3.2:1b", hidden=2048, layers=16, heads=32, kv_heads=8,
               head_dim=64, intermediate=8192, vocab=128256),
     "llama3.2-1b")
_reg(ModelSpec("llama3.2:3b", hidden=3072, layers=28, heads=24, kv_heads=8,
               head_dim=128, intermediate=8192, vocab=128256),
     "llama3.2", "llama3.2:latest", "llama3.2-3b")
_reg(ModelSpec("llama3:8b", hidden=4096, layers=32, heads=32, kv_heads=8,
               head_dim=128, intermediate=14336, vocab=128256,
               tie_embeddings=False),
     "llama3.1:8b", "llama3-8b", "llama3", "llama3:latest")
_reg(ModelSpec("llama3:70b", hidden=8192, layers=80, heads=64, kv_heads=8,
               head_dim=128, intermediate=28672, vocab=128256,
               tie_embeddings=False),
     "llama3.1:70b", "llama3-70b")
# Qwen2.5 family (the reference's own CI model is qwen2.5:0.5b,
# .github/workflows/integration-tests.yml:28): llama-style GQA +
# SwiGLU with q/k/v projection BIAS and rope theta 1e6
_reg(ModelSpec("qwen2.5:0.5b", hidden=896, layers=24, heads=14, kv_heads=2,
               head_dim=64, intermediate=4864, vocab=151936,
               rope_theta=1e6, norm_eps=1e-6, max_seq_len=32768,
               qkv_bias=True),
     "qwen2.5-0.5b", "qwen2.5:0.5b-instruct")
_reg(ModelSpec("qwen2.5:1.5b", hidden=1536, layers=28, heads=12, kv_heads=2,
               head_dim=128, intermediate=8960, vocab=151936,
               rope_theta=1e6, norm_eps=1e-6, max_seq_len=32768,
               qkv_bias=True),
     "qwen2.5-1.5b")
_reg(ModelSpec("qwen2.5:7b", hidden=3584, layers=28, heads=28, kv_heads=4,
               head_dim=128, intermediate=18944, vocab=152064,
               rope_theta=1e6, norm_eps=1e-6, max_seq_len=32768,
               qkv_bias=True, tie_embeddings=False),
     "qwen2.5-7b", "qwen2.5", "qwen2.5:latest")
# tiny configs for CPU tests and CI (tiny2: a SECOND architecture so
# mixed-fleet routing tests have two distinct models on CPU)
_reg(ModelSpec("tiny", hidden=256, layers=2, heads=4, kv_heads=2, head_dim=64,
               intermediate=512, vocab=512, max_seq_len=256),
     "tiny:latest")
_reg(ModelSpec("tiny2", hidden=128, layers=2, heads=2, kv_heads=2,
               head_dim=64, intermediate=256, vocab=512, max_seq_len=256),
     "tiny2:latest")
_reg(ModelSpec("tiny-qwen", hidden=128, layers=2, heads=4, kv_heads=2,
               head_dim=32, intermediate=256, vocab=512, max_seq_len=256,
               rope_theta=1e6, norm_eps=1e-6, qkv_bias=True),
     "tiny-qwen:latest")


# Birepel: xLSTM-style mLSTM layers with a few softmax-attention layers between
# them, routed experts, the last attention layer sharing an earlier one's
# weights. "tiny-birepel" for CPU tests and CI; the other has layers of a real
# model's size
def birepel_stack(name: str, *, vocab: int, hidden: int, attn: AttentionMixer,
                  rec: MlstmMixer, dense: DenseFF, routed: RoutedFF,
                  blocks: int, positions: int) -> HybridSpec:
    """A dense-fed mLSTM layer, then `blocks` times (attention, 2 x mLSTM) fed
    by experts, then the first attention layer once more."""
    layers = [LayerSpec(rec, dense)]
    for _ in range(blocks):
        layers += [LayerSpec(attn, routed)] + [LayerSpec(rec, routed)] * 2
    layers.append(LayerSpec(attn, routed, weights_of=1))
    return HybridSpec(name, vocab=vocab, hidden=hidden, layers=tuple(layers),
                      norm_eps=1e-5, positions=positions)


_reg(birepel_stack("tiny-birepel", vocab=512, hidden=128, blocks=1,
                   positions=256,
                   attn=AttentionMixer(4, 2, 32, 32, 32 ** -0.5, 0.1, 64),
                   rec=MlstmMixer(2, 32, 48, 15.0), dense=DenseFF(256, 7.0),
                   routed=RoutedFF(8, 2, 64)),
     "tiny-birepel:latest")
_reg(birepel_stack("birepel:3b", vocab=128256, hidden=3072, blocks=2,
                   positions=16384,
                   attn=AttentionMixer(24, 8, 128, 128, 128 ** -0.5, 0.1,
                                       8192),
                   rec=MlstmMixer(12, 128, 256, 15.0),
                   dense=DenseFF(8192, 7.0),
                   routed=RoutedFF(64, 8, 1024)),
     "birepel-3b")


def get_spec(name: str, max_seq_len: int = 0) -> Spec:
    key = name.strip()
    if key not in _SPECS:
        raise KeyError(f"unknown model {name!r}; known: {sorted(set(_SPECS))}")
    spec = _SPECS[key]
    if max_seq_len and max_seq_len != spec.max_seq_len:
        spec = replace(spec, max_seq_len=max_seq_len)
    return spec


def list_specs() -> list[str]:
    return sorted({s.name for s in _SPECS.values()})


def register_spec(spec: Spec, *aliases: str) -> None:
    """Register a custom architecture at runtime (tests, custom configs)."""
    _reg(spec, *aliases)


def names_for(name: str) -> list[str]:
    """Canonical name + every alias of a model — what a worker should
    advertise so clients can use any Ollama-style spelling (the reference
    advertised Ollama's full tag list, WorkerClientService.ts:129-154)."""
    spec = get_spec(name)
    return sorted({k for k, v in _SPECS.items() if v.name == spec.name})
