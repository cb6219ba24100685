"""Layered decoders: text models described by a list of layers (a mixer each, optionally a gated feed-forward or a
mixture of experts) around residual streams or one plain residual, run by libpgmi's decoder engine (pgmi_decoder_* in include/pgmi.h).

DecoderConfig is the family's configuration; a design's config.json is turned into one by its reader in
pgmi/registry.py.  DecoderEngine owns the context and weights, StateCache the per-sequence state of up to
`slots` sequences (key / value rows, scan and recurrent states, convolution taps, token ids), step() runs the next tokens
of any set of sequences -- whole prompts, portions, single tokens, of unequal lengths, in one batch -- and
generate() decodes a batch of prompts with the token picking every engine shares.
"""
from __future__ import annotations

import ctypes
from dataclasses import dataclass, field
from typing import List, Optional, Sequence

import torch

from . import _native as N
from .engine import EngineBase

MAMBA1, ATTENTION, MINGRU = 0, 1, 2
ACT_DTYPES = {"bfloat16": N.DTYPE_BF16, "float32": N.DTYPE_F32}


@dataclass
class DecoderLayer:
    mixer: int            # MAMBA1 | ATTENTION | MINGRU
    conv: int = 0         # mamba1: convolution taps, step rank, channels, states per channel
    dt_rank: int = 0
    inner: int = 0
    state: int = 0
    width: int = 0        # mingru: channels
    heads: int = 0        # attention: query heads, key/value heads, query-key size, value size, window, score factor
    kv_heads: int = 0
    dim: int = 0
    vdim: int = 0
    window: int = 0
    scale: float = 0.0
    ff: int = 0           # gated feed-forward size, 0: none
    # attention, continued
    qk_norm: int = 0        # queries and keys over their root mean square per head
    v_norm: int = 0         # values too
    proj_bias: int = 0
    distance_bias: int = 0  # r1 ln(1 + r2 distance) off the scores
    keep_first: int = 0     # the first tokens that stay visible past the window
    kv_from: int = -1       # the earlier attention layer whose keys and values this one reads, -1: its own
    softcap: float = 0.0    # score = softcap tanh(score / softcap), 0: as it is
    rot_dims: int = 0       # interleaved rotary positions on this many leading dims of q and k
    rot_base: float = 0.0
    rot_factor: float = 1.0    # frequency scaling by wavelength, rot_original 0: none
    rot_low: float = 0.0
    rot_high: float = 0.0
    rot_original: float = 0.0
    # mixture of experts (instead of ff), experts 0: none
    experts: int = 0
    identity: int = 0       # experts past them that return their input
    top: int = 0
    groups: int = 0         # groups of neighbours, of which the groups_keep best can be chosen from
    groups_keep: int = 0
    expert_ff: int = 0
    shared_ff: int = 0      # gated shared expert, 0: none


@dataclass
class DecoderConfig:
    vocab: int
    width: int
    streams: int
    norm_groups: int
    norm_eps: float
    embed_scale: float
    layers: List[DecoderLayer] = field(default_factory=list)
    plain_residual: bool = False  # one stream, x + residual_mult * sublayer, instead of hyper-connections
    residual_mult: float = 1.0
    norm_scalar: bool = False     # norms weigh with one number
    canon_taps: int = 0           # causal input convolution in front of every mixer
    bigram_buckets: int = 0       # rows of the bigram embedding (less the first token's)
    bigram_mul_prev: int = 0
    bigram_mul_cur: int = 0
    untied_head: bool = False

    def native(self, max_batch: int, act_dtype: int):
        """The C ABI's view: (pgmi_decoder_config, array of pgmi_layer_spec)."""
        c = N.DecoderConfigC(self.vocab, self.width, self.streams, self.norm_groups, len(self.layers), self.norm_eps,
                             self.embed_scale, max_batch, act_dtype, self.plain_residual, self.residual_mult,
                             self.norm_scalar, self.canon_taps, self.bigram_buckets, self.bigram_mul_prev,
                             self.bigram_mul_cur, self.untied_head)
        layers = (N.LayerSpec * len(self.layers))()
        for spec, layer in zip(layers, self.layers):
            for name, _ in N.LayerSpec._fields_:
                setattr(spec, name, getattr(layer, name))
        return c, layers


class StateCache:
    """The state slab of up to `slots` sequences of at most max_tokens tokens.  alloc() hands out a slot of length
    0, free() takes it back; what a slot held before is never read (a sequence starts at position 0)."""

    def __init__(self, engine: "DecoderEngine", slots: int, max_tokens: int):
        self.slots, self.max_tokens = int(slots), int(max_tokens)
        nbytes = engine.lib.pgmi_kv_bytes(engine.ctx, self.slots, self.max_tokens)
        if nbytes < 0:
            raise ValueError("bad state cache size")
        self.slab = torch.empty(max(256, nbytes), dtype=torch.uint8, device=engine.device)
        self.length = [0] * self.slots
        self._free = list(range(self.slots - 1, -1, -1))
        self._live = set()

    def alloc(self) -> int:
        if not self._free:
            raise MemoryError("every state slot is in use")
        s = self._free.pop()
        self._live.add(s)
        self.length[s] = 0
        return s

    def free(self, slot: int) -> None:
        if slot not in self._live:
            raise ValueError(f"slot {slot} is not in use")
        self._live.remove(slot)
        self._free.append(slot)

    def check(self, slots: Sequence[int]) -> None:
        for s in slots:
            if s not in self._live:
                raise ValueError(f"slot {s} is not in use")


class DecoderEngine(EngineBase):
    """One layered decoder on one GPU.  dtype "bfloat16": bf16 products and activations with 32-bit accumulation,
    streams, norms, scores and recurrences; "float32": everything in fp32 over the same bf16 weights."""

    def __init__(self, cfg: DecoderConfig, device=None, dtype: str = "bfloat16", max_batch: int = 64):
        if dtype not in ACT_DTYPES:
            raise ValueError(f"dtype must be one of {sorted(ACT_DTYPES)}")
        self.lib = N.lib()
        self.cfg = cfg
        self.device = torch.device("cuda", torch.cuda.current_device() if device is None else
                                   torch.device(device).index or 0)
        c, layers = cfg.native(max_batch, ACT_DTYPES[dtype])
        h = ctypes.c_void_p()
        N.check(self.lib.pgmi_decoder_create(self.device.index, ctypes.byref(c), layers, ctypes.byref(h)),
                "pgmi_decoder_create")
        self.vocab, self.max_batch = cfg.vocab, max_batch
        self._bind(h)

    def prepare(self) -> None:
        """Derived tensors (padded weight rows, joined biases); after every change of the weights."""
        torch.cuda.current_stream(self.device).synchronize()
        N.check(self.lib.pgmi_prepare(self.ctx), "pgmi_prepare")
        self.prepared = True

    def new_cache(self, slots: int, max_tokens: int) -> StateCache:
        return StateCache(self, slots, max_tokens)

    # ------------------------------------------------------------------ steps
    @staticmethod
    def _i32(v: Sequence[int]):
        return (ctypes.c_int32 * len(v))(*v)

    def _device_ids(self, tokens) -> torch.Tensor:
        t = torch.as_tensor(tokens, dtype=torch.int64)
        if t.device.type == "cpu" and t.numel() and not (0 <= int(t.min()) and int(t.max()) < self.vocab):
            raise ValueError("token id outside the vocabulary")
        return t.to(self.device).contiguous()

    def forward(self, cache: StateCache, slots: Sequence[int], tokens, lens: Sequence[int],
                want: Optional[Sequence[int]] = None, taps: Optional[torch.Tensor] = None) -> torch.Tensor:
        """The next lens[r] tokens of slots[r], packed sequence after sequence in `tokens`.  Returns fp32 logits
        (len(want), vocab) of the packed rows listed in want (default: every sequence's last).  taps: fp32
        (layers, rows, width) receives the summed streams after every layer."""
        self._ready()
        cache.check(slots)
        ids = self._device_ids(tokens).view(-1)
        lens = [int(n) for n in lens]
        if sum(lens) != ids.numel() or len(lens) != len(slots):
            raise ValueError("tokens, lens and slots do not fit each other")
        if want is None:
            want, at = [], 0
            for n in lens:
                at += n
                want.append(at - 1)
        want = [int(w) for w in want]
        if taps is not None and (taps.dtype is not torch.float32 or not taps.is_contiguous() or taps.device != self.device
                                 or tuple(taps.shape) != (len(self.cfg.layers), ids.numel(), self.cfg.width)):
            raise ValueError("taps must be a contiguous fp32 (layers, rows, width) tensor on the device")
        out = torch.empty((len(want), self.vocab), dtype=torch.float32, device=self.device)
        starts = [cache.length[s] for s in slots]
        N.check(self.lib.pgmi_decoder_forward(
            self.ctx, ids.data_ptr(), len(slots), self._i32(slots), self._i32(starts), self._i32(lens),
            cache.slab.data_ptr(), cache.slots, cache.max_tokens, self._i32(want), len(want), out.data_ptr(), N.ptr(taps),
            self._s()), "pgmi_decoder_forward")
        for s, n in zip(slots, lens):
            cache.length[s] += n
        return out

    def decode(self, cache: StateCache, slots: Sequence[int], ids: torch.Tensor, n_steps: int = 1,
               logits: torch.Tensor = None, next_ids: torch.Tensor = None, tokens: torch.Tensor = None,
               graph: bool = False) -> torch.Tensor:
        """n_steps greedy steps, one token per sequence each: ids (device int64, B) are the first step's tokens,
        next_ids (may be ids) receives every step's argmax and feeds the next, tokens (n_steps, B) records them.
        Returns the last step's fp32 logits (B, vocab)."""
        self._ready()
        cache.check(slots)
        B = len(slots)
        for t, n in ((ids, B), (next_ids, B), (tokens, n_steps * B)):
            if t is not None and (t.dtype is not torch.int64 or t.device != self.device or not t.is_contiguous()
                                  or t.numel() < n):
                raise ValueError("token tensors must be contiguous int64 tensors on the engine's device")
        if logits is None:
            logits = torch.empty((B, self.vocab), dtype=torch.float32, device=self.device)
        elif logits.dtype is not torch.float32 or not logits.is_contiguous() or logits.numel() < B * self.vocab:
            raise ValueError("logits must be a contiguous fp32 (B, vocab) tensor")
        pos = [cache.length[s] for s in slots]
        N.check(self.lib.pgmi_decoder_decode(
            self.ctx, ids.data_ptr(), B, self._i32(slots), self._i32(pos), cache.slab.data_ptr(), cache.slots,
            cache.max_tokens, n_steps, logits.data_ptr(), N.ptr(next_ids), N.ptr(tokens), int(graph), self._s()),
            "pgmi_decoder_decode")
        for s in slots:
            cache.length[s] += n_steps
        return logits

    def step(self, cache: StateCache, slots: Sequence[int], tokens: Sequence[Sequence[int]], want=None,
             graph: bool = True) -> torch.Tensor:
        """One step of a batch: tokens[r] are the next tokens of slots[r].  Logits of the packed rows in want
        (default: each sequence's last).  A step of single tokens that continue sequences runs the decode path."""
        lens = [len(t) for t in tokens]
        if all(n == 1 for n in lens) and all(cache.length[s] > 0 for s in slots):
            B = len(lens)
            buf = self._logits_buf.get(B)
            if buf is None:  # stable addresses let the captured step be replayed
                buf = self._logits_buf[B] = (torch.empty((B, self.vocab), dtype=torch.float32, device=self.device),
                                             torch.empty(B, dtype=torch.int64, device=self.device))
            logits, ids = buf
            ids.copy_(self._device_ids([t[0] for t in tokens]))
            self.decode(cache, slots, ids, logits=logits, graph=graph)
            return logits.clone() if want is None else logits[torch.tensor(list(want), device=self.device, dtype=torch.int64)]
        return self.forward(cache, slots, [t for ts in tokens for t in ts], lens, want)

    # ------------------------------------------------------------------ batched generation
    @torch.no_grad()
    def generate(self, prompts: Sequence[Sequence[int]], n_tokens: int, graph: bool = True, do_sample: bool = False,
                 temperature: float = 0.8, top_p: float = 0.9, generator: Optional[torch.Generator] = None,
                 eos_token_id: Optional[int] = None, pad_token_id: Optional[int] = None, sync_every: int = 16,
                 return_lengths: bool = False, prefill_tokens: int = 8192):
        """n_tokens for every prompt (lists of token ids of any lengths): int64 (B, n_tokens), with EngineBase's
        greedy / top-p / stop-token rules.  Prompts longer than prefill_tokens in total are read in portions."""
        B = len(prompts)
        lens = [len(p) for p in prompts]
        if B < 1 or min(lens) < 1:
            raise ValueError("every prompt needs at least one token")
        cache = self.new_cache(B, max(lens) + n_tokens)
        slots = [cache.alloc() for _ in range(B)]
        first = torch.empty((B, self.vocab), dtype=torch.float32, device=self.device)
        at = [0] * B
        while any(at[r] < lens[r] for r in range(B)):
            rows, toks, ns, room = [], [], [], prefill_tokens
            for r in range(B):
                n = min(lens[r] - at[r], room)
                if n > 0:
                    rows.append(r)
                    toks.extend(prompts[r][at[r]:at[r] + n])
                    ns.append(n)
                    at[r] += n
                    room -= n
            done = [k for k, r in enumerate(rows) if at[r] == lens[r]]
            last = [sum(ns[:k + 1]) - 1 for k in done]
            lg = self.forward(cache, [slots[r] for r in rows], toks, ns, want=last)
            for k, row in zip(done, lg):
                first[rows[k]] = row

        def decode_one(cur, t, step_logits, next_ids):
            self.decode(cache, slots, cur, logits=step_logits, next_ids=next_ids, graph=graph)

        def decode_many(cur, t, n, step_logits, rec):
            self.decode(cache, slots, cur, n_steps=n, logits=step_logits, next_ids=cur, tokens=rec, graph=graph)

        return self._generate_loop(first, n_tokens, decode_one, decode_many, graph, do_sample, temperature, top_p,
                                   generator, eos_token_id, pad_token_id, sync_every, return_lengths)
