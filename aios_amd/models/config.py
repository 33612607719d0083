"""Model architecture configs for the Llama-family decoders the runtime serves.

Reference roles:
  * TinyLlama-1.1B-Chat   — operational tier (`scripts/download-models.sh:70-72`)
  * Mistral-7B-Instruct   — tactical tier    (`scripts/download-models.sh:75-77`)
  * Qwen3-8B / Qwen3-14B  — tactical/strategic routing candidates
                             (`runtime/src/model_manager.rs:471-492`)
  * Llama-3-70B           — local strategic tier, TP=8

At load time the values are read from the GGUF metadata (`from_gguf`); the
presets here are used to emit random-init synthetic GGUF files of the named
shapes (no network: checkpoints cannot be downloaded).
"""
from __future__ import annotations

import dataclasses
from typing import Dict, Optional, Tuple

from ..gguf.quants import GGMLType

ROPE_NORM = 0   # llama/mistral GGUF: adjacent pairs (x[2i], x[2i+1]) (converter pre-permutes Q/K)
ROPE_NEOX = 2   # qwen: (x[i], x[i + rot/2])


@dataclasses.dataclass(frozen=True)
class LinConfig:
    """A linear recurrence with a matrix state (csrc/layered.h LinSpec)."""
    heads: int = 1
    groups: int = 1                # of heads that share B and C (mamba2) or a query and a key (delta)
    dim: int = 64                  # state rows (key channels) per head
    vdim: int = 64                 # state columns per head
    conv: int = 4                  # taps (mamba2, delta)
    norm_groups: int = 1           # parts of the gated norm (mamba2)
    rank: int = 8                  # width of the decay's first projection (gla)
    tau: float = 1.0               # root taken of the decay (gla)


@dataclasses.dataclass(frozen=True)
class LayerConfig:
    """One layer of a model described layer by layer (csrc/layered.h LayerSpec)."""
    # "latent" attention | "mingru" | "gqa" attention | "mamba2" | "gla" | "delta" (gated delta rule)
    mixer: str = "latent"
    # a second mixer reading the same input ("mamba2" | "gla" | "delta"; "": none): mixer_scale * first + beside_scale * second
    beside: str = ""
    mixer_scale: float = 1.0
    beside_scale: float = 1.0
    lin: Optional[LinConfig] = None  # sizes of the linear recurrence among the two
    # parallel: mixer and MLP read one norm and are added together; else one after the other, each with a norm
    # of its own before it, and (post_norm) after it, and (resid_gate) its result times sigmoid(W h + b)
    parallel: bool = True
    norm_scalar: bool = False      # those norms have one number for all columns
    post_norm: bool = False
    resid_gate: bool = False
    heads: int = 1
    dim: int = 64                  # (unrotated) query-key dimensions per head
    vdim: int = 64                 # value dimensions per head
    kv_rank: int = 64              # width of the cached latent
    rot_dim: int = 0               # rotated query-key dimensions; their key part is shared by all heads
    rot_dims: int = 0              # of which the first so many turn
    rot_base: float = 10000.0
    window: int = 0                # keys a token sees, itself included; 0: all before it
    scale: float = 0.125           # of q . k
    sink: bool = True              # a learned logit per head in the softmax's denominator
    sink_one: bool = False         # gqa: one (the logit 0) in the denominator instead
    kv_heads: int = 1              # key / value heads (gqa), whose first rot_dims dimensions turn in halves
    chunk: int = 0                 # gqa: keys before a token's chunk of so many positions are out; 0: no chunks
    softcap: float = 0.0           # gqa: of the scores; 0: none
    attn_bias: bool = False        # gqa: biases of q, k, v and (out_bias) the output projection
    out_bias: bool = True
    qk_norm: bool = False          # gqa: RMS norm of all of a token's queries at once, and of all its keys
    v_norm: bool = False           # gqa: every head's value divided by its root mean square
    head_temp: bool = False        # gqa: a learned number per head multiplies its scores
    # gqa: from the second such layer on, values are mixed with the first such layer's by a learned number
    v_mix: bool = False
    out_gate: str = "element"      # head outputs times sigmoid(Wg h): "none" | "element" | "head" (one number)
    width: int = 64                # of the state (mingru)
    ff: int = 256                  # hidden width of the MLP, or of every expert; 0: none
    gated: bool = True             # the MLP has a gate; else W_down act(W_up h + b) + b
    act: str = "gelu_tanh"         # of the gate or the hidden layer: "gelu_tanh" | "silu" | "relu2", "xielu" (no gate)
    mlp_bias: bool = False         # without a gate
    mlp_scale: float = 1.0         # of the result, without a gate
    experts: int = 0               # mixture of experts (0: a dense MLP), of which every token uses `top`
    top: int = 0
    router_scale: float = 1.0
    correction: bool = False       # a learned number per expert joins the choice, not the weights
    shared_ff: int = 0             # hidden width of the expert every token runs; 0: none
    weights_of: int = -1           # layer whose weights this one uses, or -1


@dataclasses.dataclass
class ModelConfig:
    name: str
    arch: str = "llama"
    vocab_size: int = 32000
    d_model: int = 2048
    n_layers: int = 22
    n_heads: int = 32
    n_kv_heads: int = 4
    head_dim: int = 64
    d_ff: int = 5632
    rope_theta: float = 10000.0
    rope_mode: int = ROPE_NORM
    norm_eps: float = 1e-5
    max_ctx: int = 2048
    tie_embeddings: bool = False
    qk_norm: bool = False          # Qwen3
    qkv_bias: bool = False         # Qwen2
    bos_id: int = 1
    eos_id: int = 2
    tokenizer_model: str = "llama"  # "llama" (SPM) or "gpt2" (byte-level BPE)
    chat_template: str = "zephyr"
    # models described layer by layer; empty: a llama-family decoder of the sizes above
    layers: Tuple[LayerConfig, ...] = ()
    learned_pos: bool = True       # a table of max_ctx learned positions
    embed_scale: float = 1.0       # of the token embedding
    logit_scale: float = 1.0
    # embedding of token pairs, row (previous * mul_prev + current * mul_cur) mod buckets: (buckets, mul_prev, mul_cur)
    bigram: Optional[Tuple[int, int, int]] = None
    loop: Optional[Tuple[int, int, int]] = None  # layers [start, stop) run `times` times: (start, stop, times)
    # how a pass of the loop is entered: False: every pass by a projection of the residual and the embedding; True:
    # every pass but the first by adding the embedding
    loop_add: bool = False

    @property
    def q_dim(self) -> int:
        return self.n_heads * self.head_dim

    @property
    def kv_dim(self) -> int:
        return self.n_kv_heads * self.head_dim

    @property
    def qkv_dim(self) -> int:
        return self.q_dim + 2 * self.kv_dim

    def n_params(self) -> int:
        if self.layers:
            return self._layered_params()
        per_layer = self.d_model * (self.qkv_dim + self.q_dim) + 3 * self.d_model * self.d_ff + 2 * self.d_model
        emb = self.vocab_size * self.d_model * (1 if self.tie_embeddings else 2)
        return self.n_layers * per_layer + emb + self.d_model

    def _layered_params(self) -> int:
        d = self.d_model
        n = 2 * self.vocab_size * d + (self.max_ctx * d if self.learned_pos else 0)
        n += (self.bigram[0] + 1) * d if self.bigram else 0
        n += 2 * d * d + self.loop[2] * d if self.loop and not self.loop_add else 0
        for l in self.layers:
            if l.weights_of >= 0:
                continue
            for kind in (l.mixer, l.beside):
                if kind == "mamba2":
                    inner, gn = l.lin.heads * l.lin.vdim, 2 * l.lin.groups * l.lin.dim
                    n += d * (3 * inner + gn + l.lin.heads) + (inner + gn) * (l.lin.conv + 1) + inner
                elif kind == "delta":
                    nk, nv = l.lin.groups * l.lin.dim, l.lin.heads * l.lin.vdim
                    n += d * (2 * nk + 3 * nv + 2 * l.lin.heads) + (2 * nk + nv) * l.lin.conv
                elif kind == "gla":
                    nk, nv = l.lin.heads * l.lin.dim, l.lin.heads * l.lin.vdim
                    n += d * (2 * nk + 3 * nv + l.lin.rank) + nk * (l.lin.rank + 1)
            if l.mixer == "mingru":
                n += 4 * l.width * d
            elif l.mixer == "gqa":
                n += d * (l.heads + l.kv_heads) * (l.dim + l.vdim) + d * (l.heads if l.out_gate == "head" else 0)
            elif l.mixer == "latent":
                gate = {"none": 0, "element": l.heads * l.vdim, "head": l.heads}[l.out_gate]
                n += d * (l.heads * (l.dim + l.rot_dim + l.vdim) + gate + l.kv_rank + l.rot_dim)
                n += l.kv_rank * l.heads * (l.dim + l.vdim)
            if l.resid_gate:
                n += d * d * (2 if l.ff else 1)
            n += (3 if l.gated else 2) * d * (l.ff * max(1, l.experts) + l.shared_ff) + l.experts * d
        return n

    def scaled(self, **kw) -> "ModelConfig":
        return dataclasses.replace(self, **kw)

    # ------------------------------------------------------------------------------
    @classmethod
    def from_gguf(cls, reader, name: Optional[str] = None) -> "ModelConfig":
        arch = reader.architecture
        g = reader.arch_get
        d = int(g("embedding_length"))
        nh = int(g("attention.head_count"))
        nkv = int(g("attention.head_count_kv", nh))
        hd = int(g("attention.key_length", d // nh))
        tokens = reader.get("tokenizer.ggml.tokens")
        vocab = int(g("vocab_size", len(tokens) if tokens is not None else 32000))
        tmpl = reader.get("tokenizer.chat_template")
        return cls(
            name=name or str(reader.get("general.name", "model")),
            arch=arch,
            vocab_size=vocab,
            d_model=d,
            n_layers=int(g("block_count")),
            n_heads=nh,
            n_kv_heads=nkv,
            head_dim=hd,
            d_ff=int(g("feed_forward_length")),
            rope_theta=float(g("rope.freq_base", 10000.0)),
            rope_mode=ROPE_NEOX if arch in ("qwen2", "qwen3", "qwen2moe", "phi3", "gptneox") else ROPE_NORM,
            norm_eps=float(g("attention.layer_norm_rms_epsilon", 1e-5)),
            max_ctx=int(g("context_length", 2048)),
            tie_embeddings="output.weight" not in reader.tensors,
            qk_norm="blk.0.attn_q_norm.weight" in reader.tensors,
            qkv_bias="blk.0.attn_q.bias" in reader.tensors,
            bos_id=int(reader.get("tokenizer.ggml.bos_token_id", 1)),
            eos_id=int(reader.get("tokenizer.ggml.eos_token_id", 2)),
            tokenizer_model=str(reader.get("tokenizer.ggml.model", "llama")),
            chat_template=tmpl if isinstance(tmpl, str) else "zephyr",
        )


def _gefazen(name: str, vocab: int, width: int, n_layers: int, max_ctx: int, **layer) -> ModelConfig:
    l = LayerConfig(scale=layer["dim"] ** -0.5, **layer)
    return ModelConfig(name=name, arch="gefazen", vocab_size=vocab, d_model=width, n_layers=n_layers, n_heads=l.heads,
                       n_kv_heads=1, head_dim=l.dim, d_ff=l.ff, max_ctx=max_ctx, bos_id=-1, eos_id=-1,
                       layers=(l,) * n_layers)


def _movalorn(name: str, vocab: int, width: int, n_layers: int, ff: int, experts: int, top: int, expert_ff: int,
              window: int, loop: Tuple[int, int, int], max_ctx: int, state: int, **attn) -> ModelConfig:
    """Every third layer latent attention, the others minGRU; the first MLP dense, then experts."""
    common = dict(parallel=False, norm_scalar=True, post_norm=True, resid_gate=True, sink=False, out_gate="head")
    dense = dict(ff=ff, act="gelu_tanh")
    moe = dict(ff=expert_ff, act="silu", experts=experts, top=top, router_scale=1.2, correction=True, shared_ff=expert_ff)
    layers = []
    for i in range(n_layers):
        mlp = dense if i == 0 else moe
        if i % 3 == 1:
            layers.append(LayerConfig(mixer="latent", window=window, scale=(attn["dim"] + attn["rot_dim"]) ** -0.5,
                                      rot_dims=attn["rot_dim"], **attn, **common, **mlp))
        else:
            layers.append(LayerConfig(mixer="mingru", width=state, **common, **mlp))
    return ModelConfig(name=name, arch="movalorn", vocab_size=vocab, d_model=width, n_layers=n_layers,
                       n_heads=attn["heads"], n_kv_heads=1, head_dim=attn["dim"] + attn["rot_dim"], d_ff=ff, max_ctx=max_ctx,
                       bos_id=-1, eos_id=-1, layers=tuple(layers), learned_pos=False, embed_scale=0.7, logit_scale=0.4,
                       bigram=(4 * vocab + 1, 37, 11), loop=loop)


def _sinisun(name: str, vocab: int, width: int, n_layers: int, ff: int, loop: Optional[Tuple[int, int, int]], max_ctx: int,
             ssm: LinConfig, gla: LinConfig, **attn) -> ModelConfig:
    """Every third layer attention beside gated linear attention, the others Mamba-2."""
    mlp = dict(parallel=False, ff=ff, gated=False, act="relu2", mlp_bias=True)
    side = LayerConfig(mixer="gqa", beside="gla", mixer_scale=0.8, beside_scale=0.6, lin=gla, out_gate="head", attn_bias=True,
                       rot_base=5e5, scale=attn["dim"] ** -0.5, **attn, **mlp)
    ssm_layer = LayerConfig(mixer="mamba2", lin=ssm, sink=False, out_gate="none", **mlp)
    return ModelConfig(name=name, arch="sinisun", vocab_size=vocab, d_model=width, n_layers=n_layers, n_heads=attn["heads"],
                       n_kv_heads=attn["kv_heads"], head_dim=attn["dim"], d_ff=ff, max_ctx=max_ctx, bos_id=-1, eos_id=-1,
                       layers=tuple(side if i % 3 == 1 else ssm_layer for i in range(n_layers)), learned_pos=False, loop=loop,
                       loop_add=True)


def _seledra(name: str, vocab: int, width: int, n_layers: int, ff: int, max_ctx: int, delta: LinConfig, **attn) -> ModelConfig:
    """Every third layer attention, the others the gated delta rule."""
    mlp = dict(parallel=False, ff=ff, gated=False, act="xielu", mlp_scale=0.7, mixer_scale=0.7)
    att = LayerConfig(mixer="gqa", sink=False, sink_one=True, out_gate="head", attn_bias=True, out_bias=False, qk_norm=True, v_norm=True,
                      head_temp=True, v_mix=True, scale=attn["dim"] ** -0.5, **attn, **mlp)
    rec = LayerConfig(mixer="delta", lin=delta, sink=False, out_gate="none", **mlp)
    return ModelConfig(name=name, arch="seledra", vocab_size=vocab, d_model=width, n_layers=n_layers, n_heads=attn["heads"],
                       n_kv_heads=attn["kv_heads"], head_dim=attn["dim"], d_ff=ff, max_ctx=max_ctx, bos_id=-1, eos_id=-1,
                       layers=tuple(att if i % 3 == 1 else rec for i in range(n_layers)))


PRESETS: Dict[str, ModelConfig] = {
    "tinyllama-1.1b": ModelConfig(
        name="tinyllama-1.1b", vocab_size=32000, d_model=2048, n_layers=22, n_heads=32, n_kv_heads=4,
        head_dim=64, d_ff=5632, rope_theta=10000.0, max_ctx=2048, chat_template="zephyr"),
    "mistral-7b": ModelConfig(
        name="mistral-7b", vocab_size=32000, d_model=4096, n_layers=32, n_heads=32, n_kv_heads=8,
        head_dim=128, d_ff=14336, rope_theta=1e6, max_ctx=32768, chat_template="mistral"),
    "llama3-70b": ModelConfig(
        name="llama3-70b", vocab_size=128256, d_model=8192, n_layers=80, n_heads=64, n_kv_heads=8,
        head_dim=128, d_ff=28672, rope_theta=5e5, max_ctx=8192, bos_id=128000, eos_id=128009,
        tokenizer_model="gpt2", chat_template="llama3"),
    "llama3-8b": ModelConfig(
        name="llama3-8b", vocab_size=128256, d_model=4096, n_layers=32, n_heads=32, n_kv_heads=8,
        head_dim=128, d_ff=14336, rope_theta=5e5, max_ctx=8192, bos_id=128000, eos_id=128009,
        tokenizer_model="gpt2", chat_template="llama3"),
    "qwen3-8b": ModelConfig(
        name="qwen3-8b", arch="qwen3", vocab_size=151936, d_model=4096, n_layers=36, n_heads=32,
        n_kv_heads=8, head_dim=128, d_ff=12288, rope_theta=1e6, rope_mode=ROPE_NEOX, norm_eps=1e-6,
        max_ctx=32768, qk_norm=True, bos_id=151643, eos_id=151645, tokenizer_model="gpt2",
        chat_template="chatml"),
    "qwen3-14b": ModelConfig(
        name="qwen3-14b", arch="qwen3", vocab_size=151936, d_model=5120, n_layers=40, n_heads=40,
        n_kv_heads=8, head_dim=128, d_ff=17408, rope_theta=1e6, rope_mode=ROPE_NEOX, norm_eps=1e-6,
        max_ctx=32768, qk_norm=True, bos_id=151643, eos_id=151645, tokenizer_model="gpt2",
        chat_template="chatml"),
    # small shapes for unit tests (K dims multiples of 256 so every K-quant applies)
    "test-tiny": ModelConfig(
        name="test-tiny", vocab_size=512, d_model=256, n_layers=2, n_heads=4, n_kv_heads=2, head_dim=64,
        d_ff=512, rope_theta=10000.0, max_ctx=256),
    "test-small": ModelConfig(
        name="test-small", vocab_size=1024, d_model=512, n_layers=3, n_heads=8, n_kv_heads=2,
        head_dim=64, d_ff=1536, rope_theta=10000.0, max_ctx=512),
    # smallest llama-3-style shape that shards over TP=2/4/8 in whole Q4_K blocks (8 KV heads,
    # q_dim/8 and d_ff/8 multiples of 256) -- the TP tests' stand-in for Llama-3-70B
    "test-tp8-shape": ModelConfig(
        name="test-tp8-shape", vocab_size=1024, d_model=2048, n_layers=2, n_heads=16, n_kv_heads=8,
        head_dim=128, d_ff=4096, rope_theta=5e5, max_ctx=512),
    # the router's other families at test size, full vocabularies and tokenizers:
    # Qwen3 (NeoX RoPE, QK-norm, 151,936-token byte-level BPE) and Llama-3 (128,256-token BPE)
    "test-qwen3-shape": ModelConfig(
        name="test-qwen3-shape", arch="qwen3", vocab_size=151936, d_model=512, n_layers=2, n_heads=4, n_kv_heads=1,
        head_dim=128, d_ff=1536, rope_theta=1e6, rope_mode=ROPE_NEOX, norm_eps=1e-6, max_ctx=512, qk_norm=True,
        bos_id=151643, eos_id=151645, tokenizer_model="gpt2", chat_template="chatml"),
    "test-llama3-shape": ModelConfig(
        name="test-llama3-shape", vocab_size=128256, d_model=512, n_layers=2, n_heads=4, n_kv_heads=1, head_dim=128,
        d_ff=1536, rope_theta=5e5, max_ctx=512, bos_id=128000, eos_id=128009, tokenizer_model="gpt2",
        chat_template="llama3"),
    # Gefazen at the widths of the two tiers above (random-init only): TinyLlama's and Mistral-7B's
    # width, depth, heads and MLP, a 512-wide latent
    "gefazen-1b": _gefazen("gefazen-1b", 32000, 2048, 22, 4096, heads=32, dim=64, vdim=64, kv_rank=512, ff=5632),
    "gefazen-7b": _gefazen("gefazen-7b", 32000, 4096, 32, 32768, heads=32, dim=128, vdim=128, kv_rank=512, ff=14336),
    "test-gefazen": _gefazen("test-gefazen", 700, 512, 3, 512, heads=4, dim=64, vdim=32, kv_rank=64, ff=1024),
    # Movalorn at the same widths, depths and active MLP sizes (layer runs, of which a loop repeats some)
    "movalorn-1b": _movalorn("movalorn-1b", 32000, 2048, 18, 5632, 16, 3, 1408, 1024, (4, 8, 2), 4096, 2048, heads=32,
                             dim=64, vdim=64, kv_rank=512, rot_dim=32),
    "movalorn-7b": _movalorn("movalorn-7b", 32000, 4096, 26, 14336, 16, 3, 3584, 2048, (4, 10, 2), 32768, 4096, heads=32,
                             dim=128, vdim=128, kv_rank=512, rot_dim=64),
    "test-movalorn": _movalorn("test-movalorn", 600, 384, 5, 512, 6, 2, 128, 50, (1, 3, 2), 512, 320, heads=3, dim=40,
                               vdim=32, kv_rank=72, rot_dim=24),
    # Sinisun at the widths and depths (layer runs) of the first two; MLPs of equal parameter count
    "sinisun-1b": _sinisun("sinisun-1b", 32000, 2048, 18, 8448, (4, 8, 2), 4096,
                           LinConfig(heads=64, vdim=64, dim=128, groups=8, norm_groups=8),
                           LinConfig(heads=16, dim=64, vdim=128, rank=16, tau=12.0), heads=32, kv_heads=4, dim=64, vdim=64, rot_dims=64,
                           chunk=1024, softcap=40.0),
    "sinisun-7b": _sinisun("sinisun-7b", 32000, 4096, 26, 21504, (4, 10, 2), 32768,
                           LinConfig(heads=128, vdim=64, dim=128, groups=8, norm_groups=8),
                           LinConfig(heads=32, dim=64, vdim=128, rank=16, tau=12.0), heads=32, kv_heads=8, dim=128, vdim=128,
                           rot_dims=128, chunk=4096, softcap=40.0),
    "test-sinisun": _sinisun("test-sinisun", 600, 384, 4, 512, (1, 3, 2), 512,
                             LinConfig(heads=4, vdim=40, dim=24, groups=2, norm_groups=5, conv=3),
                             LinConfig(heads=3, dim=40, vdim=24, rank=8, tau=9.0), heads=6, kv_heads=3, dim=48, vdim=40,
                             rot_dims=32, chunk=50, softcap=20.0),
    # as deep as the Sinisun presets are in layer runs, states and MLPs as large
    "seledra-1b": _seledra("seledra-1b", 32000, 2048, 22, 8448, 4096, LinConfig(heads=32, vdim=128, dim=128, groups=8),
                           heads=32, kv_heads=4, dim=64, vdim=64),
    "seledra-7b": _seledra("seledra-7b", 32000, 4096, 32, 21504, 8192, LinConfig(heads=64, vdim=128, dim=128, groups=16),
                           heads=32, kv_heads=8, dim=128, vdim=128),
    "test-seledra": _seledra("test-seledra", 600, 384, 4, 512, 512, LinConfig(heads=6, vdim=40, dim=24, groups=2, conv=3),
                             heads=6, kv_heads=3, dim=48, vdim=40),
    "test-mistral-shape": ModelConfig(
        name="test-mistral-shape", vocab_size=1024, d_model=1024, n_layers=2, n_heads=8, n_kv_heads=2,
        head_dim=128, d_ff=2048, rope_theta=1e6, max_ctx=512, chat_template="mistral"),
}


def get_preset(name: str) -> ModelConfig:
    key = name.lower()
    if key not in PRESETS:
        raise KeyError(f"unknown model preset {name!r}; have {sorted(PRESETS)}")
    return PRESETS[key]


# ---------------------------------------------------------------------------------------
# Quantization recipes (which ggml type each tensor gets), mirroring the public llama.cpp
# "Q4_K_M" mix: Q6_K for output + attn_v/ffn_down in "more bits" layers, Q4_K elsewhere.
# ---------------------------------------------------------------------------------------

def _use_more_bits(i: int, n: int) -> bool:
    return i < n // 8 or i >= 7 * n // 8 or (i - n // 8) % 3 == 2


def tensor_type(recipe: str, name: str, layer: int, n_layers: int) -> GGMLType:
    r = recipe.upper()
    if name.endswith("norm.weight") or name.endswith(".bias"):
        return GGMLType.F32
    if r in ("F32",):
        return GGMLType.F32
    if r in ("F16",):
        return GGMLType.F16
    if r in ("BF16",):
        return GGMLType.BF16
    if r == "Q8_0":
        return GGMLType.Q8_0
    if r == "Q4_0":
        return GGMLType.Q6_K if name == "output.weight" else GGMLType.Q4_0
    if r == "Q4_K_M":
        if name == "output.weight":
            return GGMLType.Q6_K
        if name.endswith("attn_v.weight") or name.endswith("ffn_down.weight"):
            return GGMLType.Q6_K if _use_more_bits(layer, n_layers) else GGMLType.Q4_K
        return GGMLType.Q4_K
    if r == "Q5_K_M":
        if name == "output.weight":
            return GGMLType.Q6_K
        if name.endswith("attn_v.weight") or name.endswith("ffn_down.weight"):
            return GGMLType.Q6_K if _use_more_bits(layer, n_layers) else GGMLType.Q5_K
        return GGMLType.Q5_K
    if r in ("IQ4_NL", "IQ4_XS"):  # non-linear 4-bit levels (expanded to bf16 at load)
        return GGMLType.Q6_K if name == "output.weight" else GGMLType[r]
    if r in ("Q4_1", "Q5_0", "Q5_1"):  # legacy 32-block files: expanded to bf16 at load
        return GGMLType.Q6_K if name == "output.weight" else GGMLType[r]
    if r == "Q3_K_M":  # 3-bit K-quant mix (expanded to bf16 at load, like Q2_K)
        if name == "output.weight":
            return GGMLType.Q6_K
        if name.endswith("attn_v.weight") or name.endswith("ffn_down.weight"):
            return GGMLType.Q5_K if _use_more_bits(layer, n_layers) else GGMLType.Q4_K
        return GGMLType.Q4_K if name.endswith("attn_output.weight") else GGMLType.Q3_K
    if r == "Q2_K":
        if name == "output.weight":
            return GGMLType.Q6_K
        if name.endswith("attn_v.weight") or name.endswith("ffn_down.weight"):
            return GGMLType.Q4_K if _use_more_bits(layer, n_layers) else GGMLType.Q3_K
        return GGMLType.Q2_K
    if r == "Q6_K":
        return GGMLType.Q6_K
    if r == "Q4_K":
        return GGMLType.Q4_K
    if r == "Q5_K":
        return GGMLType.Q5_K
    raise ValueError(f"unknown quant recipe {recipe}")
