"""Model architectures: presets (random-init weights of these shapes) and checkpoint folders.

Encoders (BGE / E5 class, BERT layers) replace OpenAI text-embedding-3-* (SURVEY.md §2.4 N1/N2);
decoders (Phi-3-mini / Llama-3 / Binupel / Zamitar) replace gpt-4o-mini for Summarize / Answer (N6/N7). A decoder is
named by a preset or by a folder with ``config.json`` and ``*.safetensors``, whose "architecture" picks the
parser (``ARCHITECTURES``) and thereby the model class (``models.make_decoder``).
"""
from __future__ import annotations

import os
from dataclasses import dataclass


@dataclass(frozen=True)
class EncoderConfig:
    name: str
    vocab: int = 30522
    hidden: int = 768
    layers: int = 12
    heads: int = 12
    ffn: int = 3072
    max_pos: int = 512
    type_vocab: int = 2
    eps: float = 1e-12
    pooling: str = "cls"  # "cls" (BGE) or "mean" (E5)

    @property
    def head_dim(self) -> int:
        return self.hidden // self.heads

    def param_count(self) -> int:
        h, f = self.hidden, self.ffn
        per = 4 * h * h + 2 * h * f + 9 * h + f
        return self.vocab * h + self.max_pos * h + self.type_vocab * h + 2 * h + self.layers * per


@dataclass(frozen=True)
class DecoderConfig:
    name: str
    vocab: int
    hidden: int
    layers: int
    heads: int
    kv_heads: int
    ffn: int
    max_pos: int
    rope_theta: float
    eps: float = 1e-5
    tie_embeddings: bool = False

    @property
    def head_dim(self) -> int:
        return self.hidden // self.heads

    def param_count(self) -> int:
        h, d = self.hidden, self.head_dim
        attn = h * (self.heads + 2 * self.kv_heads) * d + self.heads * d * h
        mlp = 3 * h * self.ffn
        emb = self.vocab * h * (1 if self.tie_embeddings else 2)
        return emb + self.layers * (attn + mlp + 2 * h) + h

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        return self.layers * 2 * self.kv_heads * self.head_dim * dtype_bytes


# ---------------------------------------------------------------------- decoders of mixed layers
@dataclass(frozen=True)
class GatedRecurrence:
    """Recurrent block in the manner of Griffin: gated diagonal recurrence behind a short convolution, times a branch."""
    width: int
    blocks: int   # equal parts of the channels with gate matrices of their own
    conv: int     # taps

    def param_count(self, h: int) -> int:
        w = self.width
        return 3 * h * w + w * (2 + self.conv + 1 + 1 + 2) + 2 * w * (w // self.blocks)


@dataclass(frozen=True)
class SigmoidAttention:
    """Causal attention with unnormalised sigmoid weights, normed queries and keys, values = keys."""
    heads: int
    kv_heads: int
    dim: int
    scale: float
    q_temp: tuple[float, float] | None = None  # (coef, every)

    def param_count(self, h: int) -> int:
        return h * (2 * self.heads + self.kv_heads) * self.dim + 2 * self.dim + self.heads * (1 + h)


@dataclass(frozen=True)
class SelectiveScan:
    """Mamba (selective state space) block."""
    inner: int
    state: int
    dt_rank: int
    conv: int

    def param_count(self, h: int) -> int:
        n = self.inner
        return 3 * h * n + n * (self.conv + 3 + 2 * self.dt_rank + 3 * self.state)


@dataclass(frozen=True)
class ChannelDelta:
    """Gated delta rule with a decay per key channel, behind short convolutions; low-rank decays and output gates."""
    heads: int
    kv_heads: int     # query / key heads
    dim: int          # key channels of a head
    vdim: int
    conv: int         # taps
    decay_rank: int
    gate_rank: int

    def param_count(self, h: int) -> int:
        qkv = 2 * self.kv_heads * self.dim + self.heads * self.vdim
        return (qkv * (h + self.conv) + self.heads * (h + 1) + self.vdim + self.decay_rank * (h + self.heads * self.dim)
                + self.heads * self.dim + self.gate_rank * (h + self.heads * self.vdim) + self.heads * self.vdim * h)


@dataclass(frozen=True)
class LatentAttention:
    """Softmax attention whose keys and values are read off a cached low-rank latent, beside one rotated key part
    that all heads share; a learned sink in every head's denominator; gated output."""
    heads: int
    dim: int          # unrotated query / key columns of a head
    rot_dim: int      # rotated ones
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot_base: float

    def param_count(self, h: int) -> int:
        H = self.heads
        return (self.q_rank * (h + 1 + H * (self.dim + self.rot_dim)) + (self.kv_rank + self.rot_dim) * h + self.kv_rank
                + self.kv_rank * H * (self.dim + self.vdim) + H + 2 * h * H * self.vdim)


@dataclass(frozen=True)
class HybridLayer:
    mixer: GatedRecurrence | SigmoidAttention | SelectiveScan | ChannelDelta | LatentAttention
    ff: int = 0                     # 0: no feed-forward
    weights_of: int | None = None   # use that layer's tensors (with a state of its own)


@dataclass(frozen=True)
class LayerLoop:
    """Layers ``start`` up to, not including, ``stop`` are passed through ``times`` times. A pass opens by adding a learned
    vector of its own to the stream; later passes also add the scaled embeddings again."""
    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class LayerRun:
    """One execution of a layer, with a cache or state of its own."""
    layer: int                    # whose mixer and feed-forward sizes it has
    weights: int                  # whose tensors it uses
    loop_pass: int | None = None  # this run begins that pass of the loop


@dataclass(frozen=True)
class HybridConfig:
    """A decoder whose layers mix different sequence mixers on an fp32 residual stream. ``block``:

    "postnorm"  the RMS norm after the sum, x <- norm(alpha x + sublayer(x)), mixer then feed-forward (relu-gated),
                token shift ahead of every mixer, an output head of its own
    "parallel"  one layer norm ahead of both sublayers, x <- x + s1 mixer(norm(x)) + s2 ff(norm(x)) with learned
                scales per column, silu-gated feed-forward with biases, the embedding table as output head
    """
    name: str
    vocab: int
    hidden: int
    spec: tuple[HybridLayer, ...]
    eps: float
    alpha: float = 1.0
    block: str = "postnorm"
    embed_scale: float = 1.0
    loop: LayerLoop | None = None
    max_pos: int = 1 << 20   # no learned positions: bounds the page table
    path: str = ""           # checkpoint folder ("": random init)

    @property
    def layers(self) -> int:
        """Layer executions of one token."""
        return len(self.runs)

    @property
    def runs(self) -> tuple[LayerRun, ...]:
        def run(i, loop_pass=None):
            w = self.spec[i].weights_of
            return LayerRun(i, i if w is None else w, loop_pass)
        n, lp = len(self.spec), self.loop
        if lp is None:
            return tuple(run(i) for i in range(n))
        body = [run(i, t if i == lp.start else None) for t in range(lp.times) for i in range(lp.start, lp.stop)]
        return (*(run(i) for i in range(lp.start)), *body, *(run(i) for i in range(lp.stop, n)))

    def param_count(self) -> int:
        h = self.hidden
        own = [s for s in self.spec if s.weights_of is None]
        mixers = sum(s.mixer.param_count(h) + 3 * h * s.ff for s in own)
        if self.block == "parallel":
            loop = self.loop.times * h if self.loop else 0
            return self.vocab * h + h + loop + mixers + sum(h * (3 if s.ff else 2) + 2 * s.ff + (h if s.ff else 0) for s in own)
        return 2 * self.vocab * h + h + mixers + sum(h * (3 if s.ff else 2) for s in own)

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        def per(m):
            if isinstance(m, SigmoidAttention):
                return m.kv_heads * (m.dim * dtype_bytes + 4)
            return (m.kv_rank + m.rot_dim) * dtype_bytes if isinstance(m, LatentAttention) else 0
        return sum(per(self.spec[r.layer].mixer) for r in self.runs)


def _binupel_mixer(kind: str, m: dict):
    if kind == "rglru":
        if m["width"] % m["blocks"]:
            raise ValueError(f"rglru: blocks={m['blocks']} must divide width={m['width']}")
        return GatedRecurrence(m["width"], m["blocks"], m["conv"])
    if kind == "attention":
        if m["heads"] % m["kv_heads"]:
            raise ValueError(f"attention: kv_heads={m['kv_heads']} must divide heads={m['heads']}")
        if m.get("vdim", m["dim"]) != m["dim"]:
            raise ValueError(f"attention: the values are the keys, vdim={m['vdim']} must equal dim={m['dim']}")
        t = m.get("q_temp")
        return SigmoidAttention(m["heads"], m["kv_heads"], m["dim"], float(m["scale"]),
                                (float(t["coef"]), float(t["every"])) if t else None)
    if kind == "mamba1":
        return SelectiveScan(m["inner"], m["state"], m["dt_rank"], m["conv"])
    raise ValueError(f"unknown mixer {kind!r} (rglru, attention, mamba1)")


def binupel_config(c: dict, name: str, path: str = "") -> HybridConfig:
    """The parsed ``config.json`` of a Binupel checkpoint."""
    spec = []
    for i, layer in enumerate(c["layers"]):
        mlp, src = layer.get("mlp"), layer.get("weights_of")
        if mlp and mlp.get("kind", "dense") != "dense":
            raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r} (dense)")
        spec.append(HybridLayer(_binupel_mixer(layer["type"], layer["mixer"]), mlp["ff"] if mlp else 0, src))
    for i, s in enumerate(spec):
        if s.weights_of is not None:
            j = s.weights_of
            if not 0 <= j < len(spec) or spec[j].weights_of is not None:
                raise ValueError(f"layer {i}: weights_of={j} names no layer with tensors of its own")
            if (spec[j].mixer, spec[j].ff) != (s.mixer, s.ff):
                raise ValueError(f"layer {i} differs from layer {j}, whose weights it uses")
    return HybridConfig(name, c["vocab"], c["width"], tuple(spec), float(c["norm"]["eps"]), alpha=float(c["postln_alpha"]),
                        path=path)


def _zamitar_mixer(kind: str, m: dict, rows):
    """rows(name): first dimension of one of the mixer's tensors, for the sizes that only the tensors give."""
    if kind == "channel_delta":
        if m["heads"] % m["kv_heads"]:
            raise ValueError(f"channel_delta: kv_heads={m['kv_heads']} must divide heads={m['heads']}")
        return ChannelDelta(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], rows("a1"), rows("g1"))
    if kind == "latent_attention":
        rot = m["rot"]
        if rot.get("dims", m["rot_dim"]) != m["rot_dim"] or m["rot_dim"] % 2:
            raise ValueError(f"latent_attention: rot.dims={rot.get('dims')} must be the whole, even rot_dim={m['rot_dim']}")
        return LatentAttention(m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["q_rank"], m["kv_rank"], float(m["scale"]),
                               float(rot["base"]))
    raise ValueError(f"unknown mixer {kind!r} (channel_delta, latent_attention)")


def zamitar_config(c: dict, name: str, path: str = "", shapes: dict | None = None) -> HybridConfig:
    """The parsed ``config.json`` of a Zamitar checkpoint; shapes: its tensors' (default: read from ``path``)."""
    if shapes is None:
        from .checkpoint import tensor_shapes
        shapes = tensor_shapes(path)
    spec = []
    for i, layer in enumerate(c["layers"]):
        mlp = layer.get("mlp")
        if mlp and mlp.get("kind", "dense") != "dense":
            raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r} (dense)")

        def rows(tensor, i=i):
            if f"l{i}.mix.{tensor}" not in shapes:
                raise ValueError(f"{name}: missing tensor l{i}.mix.{tensor}")
            return shapes[f"l{i}.mix.{tensor}"][0]
        spec.append(HybridLayer(_zamitar_mixer(layer["type"], layer["mixer"], rows), mlp["ff"] if mlp else 0))
    loop = c.get("loop")
    if loop:
        loop = LayerLoop(loop["start"], loop["stop"], loop["times"])
        if not (0 <= loop.start < loop.stop <= len(spec) and loop.times >= 1):
            raise ValueError(f"loop {loop.start} .. {loop.stop} x {loop.times} does not fit {len(spec)} layers")
    return HybridConfig(name, c["vocab"], c["width"], tuple(spec), float(c["norm"]["eps"]), block="parallel",
                        embed_scale=float(c["embedding"]["scale"]), loop=loop or None, path=path)


ARCHITECTURES = {"Binupel": binupel_config, "Zamitar": zamitar_config}


def _binupel(name: str, hidden: int, ff: int, vocab: int, groups: int, rec: GatedRecurrence, att: SigmoidAttention,
             ssm: SelectiveScan) -> HybridConfig:
    layer = [HybridLayer(m, ff) for m in (rec, att, ssm, ssm)]
    return HybridConfig(name, vocab, hidden, tuple(layer * groups), alpha=2.0, eps=1e-6)


def _zamitar(name: str, hidden: int, ff: int, vocab: int, groups: int, delta: ChannelDelta, att: LatentAttention,
             loop: LayerLoop | None = None) -> HybridConfig:
    layer = [HybridLayer(m, ff) for m in (delta, delta, delta, att)]
    return HybridConfig(name, vocab, hidden, tuple(layer * groups), eps=1e-6, block="parallel", embed_scale=hidden ** 0.5,
                        loop=loop)


ENCODERS = {
    "bge-small": EncoderConfig("bge-small", hidden=384, layers=12, heads=12, ffn=1536),
    "bge-base": EncoderConfig("bge-base"),
    "bge-large": EncoderConfig("bge-large", hidden=1024, layers=24, heads=16, ffn=4096),
    "e5-base": EncoderConfig("e5-base", pooling="mean"),
    "e5-large": EncoderConfig("e5-large", hidden=1024, layers=24, heads=16, ffn=4096, pooling="mean"),
    "tiny-enc": EncoderConfig("tiny-enc", vocab=30522, hidden=128, layers=2, heads=2, ffn=256, max_pos=512),
}

DECODERS = {
    "phi3-mini": DecoderConfig("phi3-mini", vocab=32064, hidden=3072, layers=32, heads=32, kv_heads=32,
                               ffn=8192, max_pos=4096, rope_theta=10000.0),
    "llama3-8b": DecoderConfig("llama3-8b", vocab=128256, hidden=4096, layers=32, heads=32, kv_heads=8,
                               ffn=14336, max_pos=8192, rope_theta=500000.0),
    "llama3-70b": DecoderConfig("llama3-70b", vocab=128256, hidden=8192, layers=80, heads=64, kv_heads=8,
                                ffn=28672, max_pos=8192, rope_theta=500000.0),
    "tiny-dec": DecoderConfig("tiny-dec", vocab=32064, hidden=256, layers=2, heads=4, kv_heads=2, ffn=512,
                              max_pos=4096, rope_theta=10000.0),
    # Llama-3-70B's TP=8 layout in miniature: 8 KV heads (one per rank), GQA group 2, FFN / vocab
    # divisible by 8 ranks (distributed tests, bench.py's TP verdict from 3 ranks); head dim 64, one
    # the GPU decode-attention kernels take
    "tiny-dec-tp8": DecoderConfig("tiny-dec-tp8", vocab=32064, hidden=1024, layers=2, heads=16, kv_heads=8,
                                  ffn=1024, max_pos=4096, rope_theta=500000.0),
    # Binupel at Llama-3-8B's width, feed-forward, attention shape and vocabulary (8 x [recurrence,
    # attention, 2 x scan]: 9.1 G parameters), and a miniature
    "binupel-9b": _binupel("binupel-9b", 4096, 14336, 128256, 8, GatedRecurrence(4096, 16, 4),
                           SigmoidAttention(32, 8, 128, 128 ** -0.5, (0.1, 8192)), SelectiveScan(8192, 16, 256, 4)),
    "tiny-binupel": _binupel("tiny-binupel", 256, 512, 32064, 1, GatedRecurrence(320, 5, 4),
                             SigmoidAttention(8, 2, 32, 32 ** -0.5, (0.1, 64)), SelectiveScan(448, 16, 24, 4)),
    # Zamitar at the same width, feed-forward and vocabulary (8 x [3 x delta rule, latent attention]), and a
    # miniature whose later layers run twice
    "zamitar-8b": _zamitar("zamitar-8b", 4096, 14336, 128256, 8, ChannelDelta(32, 32, 128, 128, 4, 128, 128),
                           LatentAttention(32, 128, 64, 128, 1536, 512, 192 ** -0.5, 500000.0)),
    "tiny-zamitar": _zamitar("tiny-zamitar", 256, 512, 32064, 1, ChannelDelta(6, 3, 32, 48, 4, 24, 40),
                             LatentAttention(4, 32, 16, 48, 96, 64, 48 ** -0.5, 10000.0), LayerLoop(1, 4, 2)),
}

ALIASES = {"text-embedding-3-large": "bge-large", "text-embedding-3-small": "bge-base",
           "gpt-4o-mini": "phi3-mini"}


def encoder_config(name: str) -> EncoderConfig:
    name = ALIASES.get(name, name)
    if name not in ENCODERS:
        raise ValueError(f"unknown encoder arch {name!r}; choose from {sorted(ENCODERS)}")
    return ENCODERS[name]


def decoder_dtypes(cfg) -> tuple[str, ...]:
    """The precisions a decoder runs in."""
    return ("bf16", "fp32") if isinstance(cfg, HybridConfig) else ("bf16",)


def checkpoint_config(path: str):
    """The configuration in a checkpoint folder's ``config.json``."""
    from .checkpoint import read_config
    c = read_config(path)
    arch = c.get("architecture")
    if arch not in ARCHITECTURES:
        raise ValueError(f"{path}: unknown architecture {arch!r}; known: {sorted(ARCHITECTURES)}")
    return ARCHITECTURES[arch](c, os.path.basename(os.path.abspath(path)), os.path.abspath(path))


def decoder_config(name: str) -> DecoderConfig | HybridConfig:
    """A preset's configuration, or that of a checkpoint folder."""
    from .checkpoint import is_checkpoint
    name = ALIASES.get(name, name)
    if name in DECODERS:
        return DECODERS[name]
    if is_checkpoint(name):
        return checkpoint_config(name)
    raise ValueError(f"unknown decoder arch {name!r}; choose from {sorted(DECODERS)} or name a checkpoint folder")
