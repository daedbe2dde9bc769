"""Model architecture registry.

The reference has no model definitions at all (compute lived in Ollama);
these specs reproduce the Llama-family architectures its deployments serve
via Ollama model tags (llama3.2:1b, llama3.2:3b,
llama3:70b).
"""

from __future__ import annotations

import glob
import json
import math
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
class Yarn:
    """YaRN: pairs that turn fewer than `slow` times within the `original`
    length turn `factor` times slower, those that turn more than `fast` times
    keep their speed, those between are interpolated; cosines and sines grow by
    0.1 ln(factor) + 1."""
    factor: float
    original: int
    fast: float
    slow: float


@dataclass(frozen=True)
class Rotary:
    """Neighbouring pairs of a head's first `dims` coordinates turn by
    p base^(-2 i / dims)."""
    base: float
    dims: int
    scaling: Optional[Yarn] = None

    def frequencies(self) -> tuple[list[float], float]:
        """Angle of each pair per position, and the factor on cosines and
        sines."""
        d, y = self.dims, self.scaling
        f = [self.base ** (-2 * i / d) for i in range(d // 2)]
        if y is None:
            return f, 1.0

        def pair(turns: float) -> float:
            return d * math.log(y.original / (2 * math.pi * turns)) \
                / (2 * math.log(self.base))

        lo = max(math.floor(pair(y.fast)), 0)
        hi = min(math.ceil(pair(y.slow)), d - 1)
        slower = [min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
                  for i in range(d // 2)]
        return [a / y.factor * r + a * (1 - r) for a, r in zip(f, slower)], \
            0.1 * math.log(y.factor) + 1


@dataclass(frozen=True)
class AttentionMixer:
    """Grouped softmax attention: rotated (if `rot`) unit-RMS q and k, a query
    temperature 1 + q_coef ln(floor((p + 1) / q_every) + 1), a sink term, an
    output gate per head or per element. With a window a query sees the last
    `window` positions, its own included, and the first keep_first."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    q_coef: float = 0.0
    q_every: int = 1
    rot: Optional[Rotary] = None
    window: int = 0                # 0: all
    keep_first: int = 0
    sink: bool = True
    gate: str = "head"             # or "element"

    def params(self, width: int) -> int:
        h, g = self.heads, self.kv_heads
        gates = h * self.vdim if self.gate == "element" else h
        return width * (h * self.dim + g * (self.dim + self.vdim) + gates
                        + h * self.vdim) + h * self.sink


@dataclass(frozen=True)
class TalkingMixer:
    """Grouped softmax attention with one projection (and bias) for keys and
    values: a value is the raw projection, a key is made from it by an RMS norm
    with a weight over the head and the rotation, so that values alone are
    cached. Queries are normed and rotated alike: pairs (i, i + rot_dims / 2) of
    the first rot_dims coordinates turn by p rot_base^(-2 i / rot_dims). Scores
    are soft-capped at `cap`; a query sees the keys of its own chunk of `chunk`
    positions; the softmax's denominator holds an extra 1; a matrix mixes the
    heads' weights."""
    heads: int
    kv_heads: int
    dim: int
    scale: float
    cap: float
    chunk: int
    rot_base: float
    rot_dims: int

    def params(self, width: int) -> int:
        h, g, d = self.heads, self.kv_heads, self.dim
        return (width + 1) * (h + g) * d + 2 * d + h * h + width * h * d


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
class LatentMixer:
    """Softmax attention whose keys and values are made from one latent per
    token (kv_rank, RMS-normed) plus a rotated key part that all heads share;
    queries go through a latent of q_rank. Only the latent and the rotated part
    are cached. Neighbouring pairs of the first rot_dims coordinates of the
    rotated part turn by p base^(-2 i / rot_dims). One output gate per head."""
    heads: int
    dim: int                       # unrotated query/key size of a head
    rot_dim: int
    vdim: int
    kv_rank: int
    q_rank: int
    scale: float
    rot_base: float
    rot_dims: int

    def params(self, width: int) -> int:
        h, k = self.heads, self.kv_rank
        return width * (self.q_rank + k + self.rot_dim + h + h * self.vdim) \
            + self.q_rank * h * (self.dim + self.rot_dim) \
            + k * h * (self.dim + self.vdim) + self.q_rank + k


@dataclass(frozen=True)
class GlaMixer:
    """Gated linear attention: a matrix memory per head whose rows decay by
    sigmoid(z)^(1/tau) per key channel, z from a projection of low rank."""
    heads: int
    dim: int
    vdim: int
    tau: float
    rank: int = 16

    def params(self, width: int) -> int:
        h = self.heads
        return width * (h * (2 * self.dim + 3 * self.vdim) + self.rank) \
            + (self.rank + 1) * h * self.dim + self.vdim


@dataclass(frozen=True)
class LightningMixer:
    """Linear attention with SiLU on q, k and v: a matrix memory per head that
    decays by a constant per token. The heads' outputs are normed together and
    gated by element."""
    heads: int
    dim: int
    vdim: int
    decay: tuple[float, ...]

    def params(self, width: int) -> int:
        return width * self.heads * (2 * self.dim + 3 * self.vdim) \
            + self.heads * self.vdim


@dataclass(frozen=True)
class ParallelMixer:
    """Attention and a recurrence on the same input; a weighted sum of their
    outputs."""
    left: AttentionMixer
    right: LightningMixer
    left_scale: float = 1.0
    right_scale: float = 1.0

    def params(self, width: int) -> int:
        return self.left.params(width) + self.right.params(width)


@dataclass(frozen=True)
class DenseFF:
    """Gated feed-forward, act(g, u) = g sigmoid(alpha g (1 + cubic g^2))
    (u + shift) with g capped at limit and u clamped to +-limit."""
    ff: int
    limit: float = math.inf
    alpha: float = 1.702
    shift: float = 1.0
    cubic: float = 0.0

    @classmethod
    def gelu_tanh(cls, ff: int) -> "DenseFF":
        """The tanh form of GELU as the gate's activation."""
        return cls(ff, alpha=2 * math.sqrt(2 / math.pi), shift=0.0,
                   cubic=0.044715)

    def params(self, width: int) -> int:
        return 3 * width * self.ff


@dataclass(frozen=True)
class PolyFF:
    """Ungated feed-forward with PolyNorm between its matrices: a polynomial of
    third degree, each power of a row divided by its own root mean square."""
    ff: int

    def params(self, width: int) -> int:
        return 2 * width * self.ff + 4


@dataclass(frozen=True)
class RoutedFF:
    """Routed experts: squared ReLU, or (gated) silu(gate) * up, or another
    unit of DenseFF's form by `unit`.

    Weights are the softmax scores of the chosen, made to sum to `scale`; with
    `sigmoid` the scores are sigmoids, and stay as they are. They multiply the
    experts' outputs, or (weigh_input) inputs. The choice is by score, plus a
    correction per expert if `corrected`, among the `keep` of `groups` equal
    groups that hold the largest ones. The last `identity` router outputs stand
    for experts that return their input. A `shared` expert takes every token,
    its output times a sigmoid gate per token."""
    experts: int
    top: int
    ff: int
    gated: bool = False
    corrected: bool = False
    groups: int = 1
    keep: int = 1
    identity: int = 0
    scale: float = 1.0
    sigmoid: bool = False
    weigh_input: bool = False
    unit: Optional[DenseFF] = None
    shared: Optional[DenseFF] = None

    @property
    def outputs(self) -> int:
        """Router outputs."""
        return self.experts + self.identity

    def params(self, width: int) -> int:
        return self.experts * width * (3 if self.gated else 2) * self.ff \
            + self.outputs * (width + self.corrected) \
            + (self.shared.params(width) + width if self.shared else 0)


@dataclass(frozen=True)
class LayerSpec:
    mixer: Union[AttentionMixer, LatentMixer, TalkingMixer, MlstmMixer,
                 GlaMixer, LightningMixer, ParallelMixer]
    ff: Union[DenseFF, PolyFF, RoutedFF, None] = None
    weights_of: Optional[int] = None
    number: Optional[int] = None   # in tensor names; None: the layer's place

    def attention(self):
        """The mixer's attention part, if any."""
        mx = self.mixer.left if isinstance(self.mixer, ParallelMixer) \
            else self.mixer
        return mx if isinstance(mx, (AttentionMixer, LatentMixer,
                                     TalkingMixer)) else None


def looped(layers: list[LayerSpec], start: int, stop: int,
           times: int) -> tuple[LayerSpec, ...]:
    """Layers in the order they run in if start .. stop - 1 run `times` times
    in a row with the same weights."""
    if not 0 <= start < stop <= len(layers) or times < 1:
        raise ValueError(f"{times} loops over layers {start} .. {stop - 1} of "
                         f"{len(layers)}")
    again = [replace(layers[i], weights_of=i) for i in range(start, stop)]
    return (*layers[:stop], *again * (times - 1),
            *(replace(ly, number=i) for i, ly in enumerate(layers)
              if i >= stop))


@dataclass(frozen=True)
class HybridSpec:
    name: str
    vocab: int
    hidden: int
    layers: tuple[LayerSpec, ...]
    norm_eps: float
    positions: int = 0             # rows of a learned position table, if any
    max_seq_len: int = 0           # 0 -> positions, or 8192 without a table
    family: str = "birepel"
    # None: x <- x + norm(y) for a sublayer's output y; else
    # x <- norm(post_alpha x + y)
    post_alpha: Optional[float] = None
    scalar_norms: bool = False     # one number per norm; else a vector, stored
    plain_norms: bool = False      # around zero, or as it is
    # a norm ahead of every sublayer, too: x <- x + norm(y(norm(x)))
    pre_norms: bool = False
    norm_groups: int = 1           # equal parts of a row, each with its own rms
    layer_scale: bool = False      # a vector on every sublayer's normed output
    embed_norm: bool = False
    # a layer passes on a weighted sum of its result, all earlier layers'
    # results and the embedding
    depth_average: bool = False
    tied: bool = True              # the head is the embedding
    logit_scale: float = 1.0
    embed_scale: float = 1.0
    # hyper-connections: this many residual streams x_s; a sublayer reads the
    # norm of sum_s in[s] x_s, then x_t <- sum_s mix[s, t] x_s + out[t] y. The
    # norm is ahead of the sublayer alone
    streams: int = 0

    def __post_init__(self) -> None:
        bound = self.positions or self.max_seq_len or 8192
        if not 0 < self.max_seq_len <= bound:
            object.__setattr__(self, "max_seq_len", bound)
        if not self.layers:
            raise ValueError(f"{self.name}: no layers")
        if self.norm_groups < 1 or self.hidden % self.norm_groups:
            raise ValueError(f"{self.name}: {self.norm_groups} norm groups of "
                             f"a width of {self.hidden}")
        if (self.norm_groups > 1 or self.layer_scale) and not self.pre_norms:
            raise ValueError(f"{self.name}: grouped norms and layer scales go "
                             "with norms on both sides")
        if self.pre_norms and (self.post_alpha is not None or
                               self.depth_average or self.embed_norm):
            raise ValueError(f"{self.name}: norms on both sides exclude norms "
                             "behind the sum, of the embedding, and depth "
                             "averages")
        if self.streams and (
                self.pre_norms or self.post_alpha is not None or
                self.depth_average or self.embed_norm or self.positions or
                self.scalar_norms or not self.plain_norms):
            raise ValueError(f"{self.name}: residual streams go with plain "
                             "norms ahead of the sublayers alone")
        if not 0 <= self.streams <= 16:
            raise ValueError(f"{self.name}: {self.streams} residual streams")
        if self.embed_scale != 1.0 and not self.streams:
            raise ValueError(f"{self.name}: a scaled embedding goes with "
                             "residual streams")
        numbers = [self.number(i) for i, ly in enumerate(self.layers)
                   if ly.weights_of is None]
        if len(set(numbers)) != len(numbers):
            raise ValueError(f"{self.name}: two layers of one number")
        for i, ly in enumerate(self.layers):
            j = self.owner(i)
            own = self.layers[j]
            if (ly.mixer, ly.ff) != (own.mixer, own.ff):
                raise ValueError(f"layer {i} uses layer {j}'s weights but "
                                 "differs from it")
            mx, ff = ly.mixer, ly.ff
            if isinstance(mx, ParallelMixer):
                _check_lightning(i, mx.right)
                mx = mx.left
            elif isinstance(mx, LightningMixer):
                _check_lightning(i, mx)
            if isinstance(mx, AttentionMixer):
                if mx.rot and (mx.rot.dims % 2 or
                               not 0 < mx.rot.dims <= mx.dim):
                    raise ValueError(f"layer {i}: rotates {mx.rot.dims} of "
                                     f"{mx.dim} dimensions")
                if mx.window < 0 or mx.keep_first < 0 or \
                        mx.gate not in ("head", "element") or \
                        mx.sink and (mx.window or mx.gate == "element"):
                    raise ValueError(
                        f"layer {i}: a window of {mx.window}, the first "
                        f"{mx.keep_first} kept, sink {mx.sink}, a gate per "
                        f"{mx.gate}")
            if isinstance(mx, (AttentionMixer, TalkingMixer)) and \
                    mx.heads % mx.kv_heads:
                raise ValueError(f"layer {i}: {mx.heads} heads over "
                                 f"{mx.kv_heads} key/value heads")
            if isinstance(mx, LatentMixer) and (
                    mx.rot_dims % 2 or not 0 <= mx.rot_dims <= mx.rot_dim):
                raise ValueError(f"layer {i}: rotates {mx.rot_dims} of "
                                 f"{mx.rot_dim} dimensions")
            if isinstance(mx, TalkingMixer):
                if mx.rot_dims % 2 or not 0 <= mx.rot_dims <= mx.dim:
                    raise ValueError(f"layer {i}: rotates {mx.rot_dims} of "
                                     f"{mx.dim} dimensions")
                if not (mx.cap > 0 and mx.chunk > 0):
                    raise ValueError(f"layer {i}: cap {mx.cap}, chunks of "
                                     f"{mx.chunk}")
            if self.pre_norms and isinstance(ff, RoutedFF):
                raise ValueError(f"layer {i}: routed experts between norms")
            if isinstance(ff, RoutedFF):
                if (ff.weigh_input or ff.unit) and not ff.gated or \
                        ff.sigmoid and (ff.corrected or ff.groups > 1 or
                                        ff.identity or ff.scale != 1.0):
                    raise ValueError(f"layer {i}: weighted inputs and units "
                                     "go with gated experts, sigmoid scores "
                                     "with a plain choice")
                if (ff.sigmoid or ff.weigh_input or ff.shared) and \
                        not self.streams:
                    raise ValueError(f"layer {i}: sigmoid scores, weighted "
                                     "inputs and shared experts go with "
                                     "residual streams")
                if ff.outputs % ff.groups or not 0 < ff.keep <= ff.groups:
                    raise ValueError(f"layer {i}: {ff.keep} of {ff.groups} "
                                     f"groups of {ff.outputs} experts")
                choice = ff.outputs // ff.groups * ff.keep
                if not 0 < ff.top <= choice:
                    raise ValueError(f"layer {i}: top {ff.top} of {choice}")

    def number(self, i: int) -> int:
        """Layer i's number in tensor names."""
        n = self.layers[i].number
        return i if n is None else n

    def owner(self, i: int) -> int:
        """The layer whose tensors layer i uses (itself, usually)."""
        seen = {i}
        while (j := self.layers[i].weights_of) is not None:
            if not 0 <= j < len(self.layers) or j in seen:
                raise ValueError(f"layer {i}: weights_of {j}")
            seen.add(j)
            i = j
        return i

    def model_info(self) -> dict:
        """Ollama-style model_info of /api/show."""
        attn = [mx for ly in self.layers if (mx := ly.attention())]
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
                     f"{f}.attention.head_count_kv":
                         getattr(attn[0], "kv_heads", attn[0].heads)}
            if isinstance(attn[0], LatentMixer):
                info |= {f"{f}.attention.kv_lora_rank": attn[0].kv_rank,
                         f"{f}.attention.q_lora_rank": attn[0].q_rank,
                         f"{f}.rope.dimension_count": attn[0].rot_dims,
                         f"{f}.rope.freq_base": attn[0].rot_base}
            elif isinstance(attn[0], TalkingMixer):
                info |= {f"{f}.attention.chunk_size": attn[0].chunk,
                         f"{f}.attention.logit_softcapping": attn[0].cap,
                         f"{f}.rope.dimension_count": attn[0].rot_dims,
                         f"{f}.rope.freq_base": attn[0].rot_base}
            else:
                if attn[0].window:
                    info[f"{f}.attention.sliding_window"] = attn[0].window
                if attn[0].rot:
                    info |= {f"{f}.rope.dimension_count": attn[0].rot.dims,
                             f"{f}.rope.freq_base": attn[0].rot.base}
        if routed:
            info |= {f"{f}.expert_count": routed[0].experts,
                     f"{f}.expert_used_count": routed[0].top}
        return info

    @property
    def params(self) -> int:
        w = self.hidden
        norm = 1 if self.scalar_norms else w
        sub = norm * (1 + self.pre_norms) + w * self.layer_scale
        total = (self.vocab * (1 if self.tied else 2) + self.positions) * w
        total += norm * (1 + self.embed_norm)
        for i, ly in enumerate(self.layers):
            if self.depth_average:
                total += i + 2
            if ly.weights_of is None:
                total += ly.mixer.params(w) + sub
                if ly.ff is not None:
                    total += ly.ff.params(w) + sub
                total += (2 + self.streams) * self.streams * (
                    1 if ly.ff is None else 2)
        return total


def _check_lightning(i: int, mx: LightningMixer) -> None:
    if len(mx.decay) != mx.heads or not all(0 <= d <= 1 for d in mx.decay):
        raise ValueError(f"layer {i}: decays {mx.decay} of {mx.heads} heads")


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


def read_birepel(cfg: dict, name: str = "birepel", shape=None) -> HybridSpec:
    """Birepel's config.json -> spec."""
    layers = tuple(
        LayerSpec(mixer=_read_mixer(ly["type"], ly["mixer"]),
                  ff=_read_ff(ly.get("mlp")), weights_of=ly.get("weights_of"))
        for ly in cfg["layers"])
    return HybridSpec(name=name, vocab=cfg["vocab"], hidden=cfg["width"],
                      layers=layers, norm_eps=float(cfg["norm"]["eps"]),
                      positions=cfg["max_positions"])


def _read_maferax_layer(i: int, ly: dict, shape) -> LayerSpec:
    _take(ly, f"layer {i}", ("type", "mixer"), ("mlp",))
    kind, d, ff = ly["type"], ly["mixer"], ly.get("mlp")
    if kind == "latent_attention":
        _take(d, kind, ("heads", "dim", "rot_dim", "vdim", "kv_rank",
                        "q_rank", "scale", "rot"))
        rot = _take(d["rot"], "rot", ("base", "dims"))
        mixer = LatentMixer(
            heads=d["heads"], dim=d["dim"], rot_dim=d["rot_dim"],
            vdim=d["vdim"], kv_rank=d["kv_rank"], q_rank=d["q_rank"],
            scale=float(d["scale"]), rot_base=float(rot["base"]),
            rot_dims=rot["dims"])
    elif kind == "gla":
        _take(d, kind, ("heads", "dim", "vdim", "tau"))
        a1 = shape(f"l{i}.mix.a1") if shape else None
        mixer = GlaMixer(heads=d["heads"], dim=d["dim"], vdim=d["vdim"],
                         tau=float(d["tau"]), **({"rank": a1[0]} if a1 else {}))
    else:
        raise ValueError(f"config: unknown mixer {kind!r}")
    if ff is None:
        return LayerSpec(mixer)
    if ff.get("kind") == "dense":
        _take(ff, "dense mlp", ("kind", "ff"))
        return LayerSpec(mixer, DenseFF.gelu_tanh(ff["ff"]))
    if ff.get("kind") != "moe":
        raise ValueError(f"config: unknown mlp kind {ff.get('kind')!r}")
    _take(ff, "moe mlp", ("kind", "expert", "router"))
    _take(ff["expert"], "expert", ("ff",))
    r = _take(ff["router"], "router", ("experts", "top"),
              ("groups", "identity", "scale"))
    g = _take(r.get("groups") or {"count": 1, "keep": 1}, "groups",
              ("count", "keep"))
    return LayerSpec(mixer, RoutedFF(
        experts=r["experts"], top=r["top"], ff=ff["expert"]["ff"], gated=True,
        corrected=True, groups=g["count"], keep=g["keep"],
        identity=r.get("identity") or 0, scale=float(r.get("scale", 1.0))))


def read_maferax(cfg: dict, name: str = "maferax", shape=None) -> HybridSpec:
    """Maferax's config.json -> spec. `shape` gives a tensor's shape, or None
    if there is no such tensor: the rank of a decay projection is not in the
    configuration."""
    _take(cfg, "model", ("layers", "vocab", "width", "norm", "postln_alpha",
                         "logit_scale"), ("architecture",))
    return HybridSpec(
        name=name, vocab=cfg["vocab"], hidden=cfg["width"],
        layers=tuple(_read_maferax_layer(i, ly, shape)
                     for i, ly in enumerate(cfg["layers"])),
        norm_eps=float(cfg["norm"]["eps"]),
        post_alpha=float(cfg["postln_alpha"]),
        logit_scale=float(cfg["logit_scale"]), **_MAFERAX)


_MAFERAX = dict(family="maferax", scalar_norms=True, embed_norm=True,
                depth_average=True, tied=False)

def _read_vivepel_layer(i: int, ly: dict) -> LayerSpec:
    _take(ly, f"layer {i}", ("type", "mixer"), ("mlp",))
    kind, d, ff = ly["type"], ly["mixer"], ly.get("mlp")
    if kind != "attention":
        raise ValueError(f"config: unknown mixer {kind!r}")
    _take(d, kind, ("heads", "kv_heads", "dim", "vdim", "scale", "softcap",
                    "rot", "mask"))
    rot = _take(d["rot"], "rot", ("base", "dims"))
    mask = _take(d["mask"], "mask", ("size",))
    if d["vdim"] != d["dim"]:
        raise ValueError(f"config: values are keys, but of size {d['vdim']}, "
                         f"not {d['dim']}")
    mixer = TalkingMixer(
        heads=d["heads"], kv_heads=d["kv_heads"], dim=d["dim"],
        scale=float(d["scale"]), cap=float(d["softcap"]),
        chunk=int(mask["size"]), rot_base=float(rot["base"]),
        rot_dims=rot["dims"])
    if ff is None:
        return LayerSpec(mixer)
    if ff.get("kind") != "dense":
        raise ValueError(f"config: unknown mlp kind {ff.get('kind')!r}")
    _take(ff, "dense mlp", ("kind", "ff"))
    return LayerSpec(mixer, PolyFF(ff["ff"]))


def read_vivepel(cfg: dict, name: str = "vivepel", shape=None) -> HybridSpec:
    """Vivepel's config.json -> spec."""
    _take(cfg, "model", ("layers", "vocab", "width", "norm"),
          ("architecture",))
    norm = _take(cfg["norm"], "norm", ("eps", "groups"))
    return HybridSpec(
        name=name, vocab=cfg["vocab"], hidden=cfg["width"],
        layers=tuple(_read_vivepel_layer(i, ly)
                     for i, ly in enumerate(cfg["layers"])),
        norm_eps=float(norm["eps"]), norm_groups=norm["groups"], **_VIVEPEL)


_VIVEPEL = dict(family="vivepel", plain_norms=True, pre_norms=True,
                layer_scale=True, tied=False)


def _read_rotary(d: dict) -> Rotary:
    _take(d, "rot", ("base", "dims"), ("scaling",))
    y = d.get("scaling")
    if y is not None:
        _take(y, "rot scaling", ("factor", "original", "fast", "slow"))
        y = Yarn(float(y["factor"]), y["original"], float(y["fast"]),
                 float(y["slow"]))
    return Rotary(float(d["base"]), d["dims"], y)


def _read_zinavik_layer(i: int, ly: dict) -> LayerSpec:
    _take(ly, f"layer {i}", ("type", "mixer"), ("mlp",))
    kind, d, ff = ly["type"], ly["mixer"], ly.get("mlp")
    if kind != "parallel":
        raise ValueError(f"config: unknown mixer {kind!r}")
    _take(d, kind, ("left", "right", "left_scale", "right_scale"))
    a = _take(d["left"], "left", ("heads", "kv_heads", "dim", "vdim", "scale",
                                  "rot", "mask"))
    b = _take(d["right"], "right", ("heads", "dim", "vdim", "decay"))
    mask = _take(a["mask"], "mask", ("size",), ("keep_first",))
    if mask["size"] < 1:
        raise ValueError(f"config: a window of {mask['size']}")
    mixer = ParallelMixer(
        AttentionMixer(heads=a["heads"], kv_heads=a["kv_heads"], dim=a["dim"],
                       vdim=a["vdim"], scale=float(a["scale"]),
                       rot=_read_rotary(a["rot"]), window=mask["size"],
                       keep_first=mask.get("keep_first") or 0, sink=False,
                       gate="element"),
        LightningMixer(b["heads"], b["dim"], b["vdim"],
                       tuple(float(x) for x in b["decay"])),
        float(d["left_scale"]), float(d["right_scale"]))
    if ff is None:
        return LayerSpec(mixer)
    if ff.get("kind") != "moe":
        raise ValueError(f"config: unknown mlp kind {ff.get('kind')!r}")
    _take(ff, "moe mlp", ("kind", "expert", "router"), ("shared",))
    e = _take(ff["expert"], "expert", ("ff", "limit"))
    r = _take(ff["router"], "router", ("experts", "top"))
    sh = ff.get("shared")
    if sh is not None:
        _take(sh, "shared expert", ("ff", "limit"))
        sh = DenseFF(sh["ff"], float(sh["limit"]))
    return LayerSpec(mixer, RoutedFF(
        experts=r["experts"], top=r["top"], ff=e["ff"],
        unit=DenseFF(e["ff"], float(e["limit"])), shared=sh, **_ZINAVIK_MOE))


_ZINAVIK = dict(family="zinavik", plain_norms=True)
_ZINAVIK_MOE = dict(gated=True, sigmoid=True, weigh_input=True)


def read_zinavik(cfg: dict, name: str = "zinavik", shape=None) -> HybridSpec:
    """Zinavik's config.json -> spec."""
    _take(cfg, "model", ("layers", "vocab", "width", "norm", "streams",
                         "embedding"), ("architecture", "loop"))
    layers = [_read_zinavik_layer(i, ly) for i, ly in enumerate(cfg["layers"])]
    loop = cfg.get("loop")
    if loop is not None:
        layers = looped(layers, **_take(loop, "loop", ("start", "stop",
                                                       "times")))
    if cfg["streams"] < 1:
        raise ValueError(f"config: {cfg['streams']} streams")
    return HybridSpec(
        name=name, vocab=cfg["vocab"], hidden=cfg["width"],
        layers=tuple(layers),
        norm_eps=float(_take(cfg["norm"], "norm", ("eps",))["eps"]),
        embed_scale=float(_take(cfg["embedding"], "embedding",
                                ("scale",))["scale"]),
        streams=cfg["streams"], **_ZINAVIK)


# "architecture" in config.json -> reader. Checkpoints without that key (HF
# layout) are loaded into the architecture that the model name gives.
_READERS: dict[str, Callable[..., Spec]] = {"Birepel": read_birepel,
                                            "Maferax": read_maferax,
                                            "Vivepel": read_vivepel,
                                            "Zinavik": read_zinavik}


def _shape_reader(path: str) -> Callable[[str], Optional[tuple]]:
    """Shapes of the tensors in a folder's safetensors files, by name."""
    def shape(name: str) -> Optional[tuple]:
        from safetensors import safe_open
        for f in sorted(glob.glob(os.path.join(path, "*.safetensors"))):
            with safe_open(f, framework="pt") as sf:
                if name in sf.keys():
                    return tuple(sf.get_slice(name).get_shape())
        return None
    return shape


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
    return _READERS[arch](cfg, name or f"{arch.lower()}:custom",
                          _shape_reader(path))


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


# Maferax: gated linear attention layers with a latent-attention layer every
# few, a dense feed-forward first and routed experts (some of them identity)
# after it, norms behind the sums, a depth average behind every layer
def maferax_stack(name: str, *, vocab: int, hidden: int, attn: LatentMixer,
                  rec: GlaMixer, dense: DenseFF, routed: RoutedFF,
                  blocks: int, alpha: float, logit_scale: float,
                  max_seq_len: int) -> HybridSpec:
    """`blocks` times (latent attention, 3 x GLA); the first layer's
    feed-forward is dense."""
    layers = []
    for _ in range(blocks):
        layers += [LayerSpec(attn, routed if layers else dense)] + \
            [LayerSpec(rec, routed)] * 3
    return HybridSpec(name, vocab=vocab, hidden=hidden, layers=tuple(layers),
                      norm_eps=1e-5, post_alpha=alpha,
                      logit_scale=logit_scale, max_seq_len=max_seq_len,
                      **_MAFERAX)


_reg(maferax_stack("tiny-maferax", vocab=512, hidden=128, blocks=1, alpha=1.7,
                   logit_scale=1.0, max_seq_len=256,
                   attn=LatentMixer(4, 32, 16, 32, 48, 64, 48 ** -0.5, 1e4,
                                    16),
                   rec=GlaMixer(2, 32, 48, 16.0, 8),
                   dense=DenseFF.gelu_tanh(256),
                   routed=RoutedFF(7, 2, 64, gated=True, corrected=True,
                                   groups=4, keep=2, identity=1, scale=1.5)),
     "tiny-maferax:latest")
_reg(maferax_stack("maferax:5b", vocab=128256, hidden=3072, blocks=2,
                   alpha=2.0, logit_scale=1.0, max_seq_len=16384,
                   attn=LatentMixer(24, 128, 64, 128, 512, 1536, 192 ** -0.5,
                                    1e5, 64),
                   rec=GlaMixer(12, 128, 256, 16.0, 16),
                   dense=DenseFF.gelu_tanh(8192),
                   routed=RoutedFF(64, 8, 1024, gated=True, corrected=True,
                                   groups=8, keep=4, identity=8, scale=2.0)),
     "maferax-5b")


# Vivepel: talking-heads attention within chunks, PolyNorm feed-forwards, norms
# in groups on both sides of every sublayer
def vivepel_stack(name: str, *, vocab: int, hidden: int, attn: TalkingMixer,
                  ff: int, layers: int, groups: int,
                  max_seq_len: int) -> HybridSpec:
    return HybridSpec(name, vocab=vocab, hidden=hidden,
                      layers=(LayerSpec(attn, PolyFF(ff)),) * layers,
                      norm_eps=1e-5, norm_groups=groups,
                      max_seq_len=max_seq_len, **_VIVEPEL)


_reg(vivepel_stack("tiny-vivepel", vocab=512, hidden=128, ff=256, layers=2,
                   groups=4, max_seq_len=256,
                   attn=TalkingMixer(4, 2, 32, 32 ** -0.5, 30.0, 48, 1e4, 16)),
     "tiny-vivepel:latest")
_reg(vivepel_stack("vivepel:2b", vocab=128256, hidden=3072, ff=12288,
                   layers=8, groups=8, max_seq_len=16384,
                   attn=TalkingMixer(24, 8, 128, 128 ** -0.5, 30.0, 4096, 5e5,
                                     64)),
     "vivepel-2b")


# Zinavik: window attention and lightning attention side by side, sigmoid-routed
# experts beside a shared one, hyper-connections, layers that run more than once
def zinavik_stack(name: str, *, vocab: int, hidden: int, mixer: ParallelMixer,
                  experts: int, top: int, ff: int, shared: int, limit: float,
                  layers: int, loop: tuple[int, int, int], streams: int,
                  max_seq_len: int) -> HybridSpec:
    routed = RoutedFF(experts, top, ff, unit=DenseFF(ff, limit),
                      shared=DenseFF(shared, limit), **_ZINAVIK_MOE)
    return HybridSpec(name, vocab=vocab, hidden=hidden,
                      layers=looped([LayerSpec(mixer, routed)] * layers, *loop),
                      norm_eps=1e-5, embed_scale=hidden ** 0.5,
                      streams=streams, max_seq_len=max_seq_len, **_ZINAVIK)


_reg(zinavik_stack("tiny-zinavik", vocab=512, hidden=128, experts=8, top=2,
                   ff=64, shared=64, limit=7.0, layers=3, loop=(1, 2, 2),
                   streams=2, max_seq_len=256,
                   mixer=ParallelMixer(
                       AttentionMixer(4, 2, 32, 32, 32 ** -0.5, window=48,
                                      keep_first=4, sink=False, gate="element",
                                      rot=Rotary(1e4, 16, Yarn(2.0, 128, 32.0,
                                                               1.0))),
                       LightningMixer(2, 32, 48, (0.9, 0.99)))),
     "tiny-zinavik:latest")
_reg(zinavik_stack("zinavik:4b", vocab=128256, hidden=3072, experts=64, top=7,
                   ff=1024, shared=1024, limit=7.0, layers=6, loop=(2, 4, 2),
                   streams=4, max_seq_len=16384,
                   mixer=ParallelMixer(
                       AttentionMixer(24, 8, 128, 128, 128 ** -0.5,
                                      window=2048, keep_first=64, sink=False,
                                      gate="element",
                                      rot=Rotary(5e5, 128, Yarn(4.0, 4096,
                                                                32.0, 1.0))),
                       LightningMixer(12, 128, 256, tuple(
                           1 - 2.0 ** (-5 - 7 * h / 11) for h in range(12))),
                       0.5, 0.5)),
     "zinavik-4b")


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
