"""Models whose layers are listed one by one, run by the native layer stack (csrc/layer_stack.hip) over paged caches and recurrent state.

A design's module (models/taduzen, models/kodupel, models/bezutar, models/lagelorn) reads its config.json and packs its checkpoint into `pie_stack_layer` descriptions; this class is what every such
model shares with the engines: the cache protocol (make_cache, enable_paged_kv), the calling convention (`model(inputs, cache=)`), the greedy fast
path (`step`) and the multi-sequence passes (`step_batch`, `prefill_batch`, `step_mixed`, `step_portions`).  Every one of them is the same pass:
rows of any sequences, each with its own position, in one batch."""
from __future__ import annotations

import ctypes as C
import math
from typing import NamedTuple

import numpy as np
import torch

from .. import _ffi
from ..cache.kv_cache import BaseCache, LatentPageAllocator, PagedLatentCache, PagedSequence, PagedStackCache, SavedLatentCache, StackPageAllocator, StackSequence
from ..cache.kv_cache.paged import TOKEN_CAPACITY_PER_PAGE

MAX_ROWS = 4096  # rows of one pass; longer prompts run as several


class Norm(NamedTuple):
    """A norm of the stack: kind PIE_NORM_*, param (DYN_TANH: alpha; RMS: eps), fp32 w and b [width rounded up to 8]."""
    kind: int
    param: float
    w: torch.Tensor
    b: torch.Tensor | None = None


class Embedding(NamedTuple):
    """What the residual starts from besides the token's vector.  streams > 0: equal copies of it (hyper-connections); positions: bf16 [rows, width] by position -- no sequence
    grows beyond them; bigram: bf16 [buckets + 1, width] by (previous token * mul_prev + token * mul_cur) mod buckets, the last row at a sequence's first token.  side: bf16 [vocab, layers *
    side size]: not part of the residual's start, but of what every layer adds to it."""
    streams: int = 0
    positions: torch.Tensor | None = None
    bigram: torch.Tensor | None = None
    mul_prev: int = 0
    mul_cur: int = 0
    side: torch.Tensor | None = None


def up8(n: int) -> int:
    return (n + 7) // 8 * 8


def pad(w: torch.Tensor, rows: int, cols: int) -> torch.Tensor:
    """w in the corner of a [rows, cols] matrix of zeros."""
    out = torch.zeros(rows, cols, dtype=w.dtype, device=w.device)
    out[:w.shape[0], :w.shape[1]] = w
    return out


def pad_head_rows(w: torch.Tensor, heads: int, n: int) -> torch.Tensor:
    """[heads * n, K] -> [heads * (n rounded up to 8), K], zero rows behind each head."""
    out = torch.zeros(heads, up8(n), w.shape[1], dtype=w.dtype, device=w.device)
    out[:, :n] = w.reshape(heads, n, -1)
    return out.flatten(0, 1)


def pad_head_columns(w: torch.Tensor, heads: int, n: int) -> torch.Tensor:
    """[N, heads * n] -> [N, heads * (n rounded up to 8)], zero columns behind each head."""
    return pad_head_rows(w.T, heads, n).T


def interleave(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
    """Rows (2 i, 2 i + 1) = (gate_i, up_i)."""
    return torch.stack([gate, up], dim=-2).flatten(-3, -2)


def yarn_frequencies(dims: int, base: float, scaling: tuple[float, float, float, float] | None = None) -> tuple[torch.Tensor, float]:
    """(fp32 [dims / 2] angle per position of every rotated pair, the factor on cos and sin).  scaling = (factor, original, fast, slow): pairs that turn
    more than `fast` times over the original context keep their frequency, pairs that turn less than `slow` times have it divided by factor, those between
    are mixed linearly (YaRN)."""
    freq = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if scaling is None:
        return torch.tensor(freq, dtype=torch.float32), 1.0
    factor, original, fast, slow = scaling
    at = lambda turns: dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))  # noqa: E731
    lo, hi = max(math.floor(at(fast)), 0), min(math.ceil(at(slow)), dims - 1)
    mix = [min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(dims // 2)]
    return torch.tensor([f * (m / factor + 1.0 - m) for f, m in zip(freq, mix)], dtype=torch.float32), 0.1 * math.log(factor) + 1.0


def pack_linear(w: torch.Tensor, dtype: torch.dtype) -> torch.Tensor:
    """A Linear weight [N, K] (bf16, device) or a batch of equal ones [B, N, K] in the stack's packed form, as bytes [B * size]."""
    w = w.to(torch.bfloat16).contiguous()
    mats = w if w.dim() == 3 else w[None]
    lib, code = _ffi.base(), _ffi.stack_dtype_code(dtype)
    n = lib.pie_stack_weight_bytes(code, mats.shape[1], mats.shape[2])
    out = torch.empty(mats.shape[0] * n, dtype=torch.uint8, device=w.device)
    for i in range(mats.shape[0]):
        mat = mats[i] if mats[i].data_ptr() % 16 == 0 else mats[i].clone()  # (a matrix of odd size starts the next one unaligned)
        _ffi.check(lib.pie_stack_pack_weight(mat.data_ptr(), mats.shape[1], mats.shape[2], code, out.data_ptr() + i * n, _ffi.stream()))
    return out


class LayerStackModel:
    def __init__(self, args, dtype: torch.dtype, width: int, vocab: int, logit_scale: float, layers: list[dict], embed: torch.Tensor, head: torch.Tensor,
                 final_norm: Norm, embed_scale: float = 1.0, embedding: Embedding = Embedding(), logit_cap: float = 0.0):
        """layers: per layer the fields of pie_stack_layer -- tensors for its pointers, Norms for its norms, dicts for structures inside it, numbers for
        the rest (absent fields are zero).  embed: bf16 [vocab, width]; head: packed."""
        self.args, self.dtype, self.width, self.vocab_size = args, dtype, width, vocab
        self.device = embed.device
        self.layers = layers
        self._held = [embed, head, final_norm, embedding]
        self.max_positions = None if embedding.positions is None else embedding.positions.shape[0]  # tokens a sequence can have
        lib = _ffi.base()
        cfg = _ffi.pie_stack_config(_ffi.stack_dtype_code(dtype), width, vocab, len(layers), logit_scale, embed_scale, embed.data_ptr(), head.data_ptr(), self._norm(final_norm), embedding.streams, self.max_positions or 0,
                                    *(None if t is None else t.data_ptr() for t in (embedding.positions, embedding.bigram)), embedding.mul_prev, embedding.mul_cur,
                                    0 if embedding.bigram is None else embedding.bigram.shape[0] - 1, logit_cap, *((None, 0) if embedding.side is None else (embedding.side.data_ptr(), embedding.side.shape[1] // len(layers))))
        self._stack = C.c_void_p()
        _ffi.check(lib.pie_stack_create(C.byref(cfg), C.byref(self._stack)))
        for i, fields in enumerate(layers):
            lay = _ffi.pie_stack_layer()
            self._fill(lay, fields)
            _ffi.check(lib.pie_stack_set_layer(self._stack, i, C.byref(lay)))
        self.row_elems = [lib.pie_stack_page_row(self._stack, i) for i in range(len(layers))]
        self.state_floats = [int(lib.pie_stack_state_floats(self._stack, i)) for i in range(len(layers))]
        self.recurrent = any(self.state_floats)
        # a latent layer's pages hold token after token; anything else is kept, shared and saved by whole pages, beside the recurrent state
        self._plain_pages = not self.recurrent and all(lay["mixer"] == _ffi.PIE_MIXER_LATENT for lay in layers)
        self.history = torch.zeros(1 << 20, dtype=torch.int32, device=self.device)  # history[p] = greedy token chosen for position p
        self._pool: LatentPageAllocator | None = None
        self._page_blocks = 16
        self._bufs: dict = {}      # per decode batch size: the persistent buffers a captured step points at
        torch.cuda.synchronize(self.device)

    @classmethod
    def _fill(cls, struct, fields: dict) -> None:
        for name, v in fields.items():
            if isinstance(v, dict):
                cls._fill(getattr(struct, name), v)
            else:
                setattr(struct, name, cls._norm(v) if isinstance(v, Norm) else v.data_ptr() if isinstance(v, torch.Tensor) else v)

    @staticmethod
    def _norm(n: Norm):
        return _ffi.pie_stack_norm(n.w.data_ptr(), None if n.b is None else n.b.data_ptr(), n.param, n.kind)

    def __del__(self):
        s = getattr(self, "_stack", None)
        if s is not None and s.value:
            try:
                _ffi.base().pie_stack_destroy(s)
            except Exception:  # noqa: BLE001  (interpreter shutdown)
                pass
            self._stack = None

    # ------------------------------------------------------------------ caches
    def _allocator(self, num_pages: int, max_sequences: int) -> LatentPageAllocator:
        if self._plain_pages:
            return LatentPageAllocator(num_pages, self.row_elems, dtype=self.dtype, device=self.device)
        return StackPageAllocator(num_pages, self.row_elems, self.state_floats, max_sequences, dtype=self.dtype, device=self.device)

    def enable_paged_kv(self, num_pages: int = 512, max_blocks: int = 16, kv_dtype: torch.dtype | None = None, kv_scales=None,
                        max_sequences: int = 32) -> LatentPageAllocator:
        """From now on make_cache() draws on one pool of `num_pages` 64-token pages (all layers) and, for recurrent layers, state slots for
        `max_sequences` live sequences.  Returns the pool."""
        if kv_dtype not in (None, self.dtype) or kv_scales is not None:
            raise ValueError(f"a layer-stack model's pages are stored in its dtype ({self.dtype})")
        self._pool = self._allocator(num_pages, max_sequences)
        self._page_blocks = max_blocks
        return self._pool

    def make_cache(self) -> list[BaseCache]:
        if self._pool is None:
            self.enable_paged_kv()
        return self.make_paged_cache(self._pool, max_blocks=self._page_blocks)

    def make_paged_cache(self, allocator: LatentPageAllocator | None = None, num_pages: int = 512, max_blocks: int = 16) -> list[BaseCache]:
        if allocator is None:
            allocator = self._allocator(num_pages, 32)
        if not isinstance(allocator, LatentPageAllocator if self._plain_pages else StackPageAllocator) or allocator.row_elems != self.row_elems or \
                allocator.dtype != self.dtype or allocator.device is None or (not self._plain_pages and allocator.state_floats != self.state_floats):
            raise ValueError("the allocator's geometry does not match this model")
        if self._plain_pages:
            seq: PagedSequence = PagedSequence(allocator, max_blocks)
            return [PagedLatentCache(seq, i) for i in range(len(self.layers))]
        seq = StackSequence(allocator, max_blocks)
        return [PagedStackCache(seq, i) for i in range(len(self.layers))]

    def adopt_cache(self, cache: list[BaseCache]) -> list[BaseCache]:
        """A cache restored from a file, copied into pages (and a state slot); anything else as it is."""
        if not isinstance(cache[0], SavedLatentCache):
            return cache
        out = self.make_cache()
        for mine, saved in zip(out, cache):
            mine.adopt(saved)
        return out

    def _sequence(self, cache: list[BaseCache]) -> PagedSequence:
        if len(cache) != len(self.layers) or not isinstance(cache[0], PagedLatentCache):
            raise TypeError("a layer-stack model runs on its own paged caches (make_cache())")
        return cache[0].page_manager

    @staticmethod
    def _sequences(seqs: list[PagedSequence]):
        a = seqs[0].allocator
        if any(s.allocator is not a for s in seqs) or len({id(s) for s in seqs}) != len(seqs):
            raise ValueError("a pass takes distinct sequences of one page pool")
        return a

    def _reserve(self, seq: PagedSequence, n: int) -> None:
        """Room for n more tokens."""
        self._check_length(seq, n)
        seq.reserve(n)

    def _check_length(self, seq: PagedSequence, n: int) -> None:
        if self.max_positions is not None and seq.offset + n > self.max_positions:
            raise ValueError(f"a sequence of {seq.offset + n} tokens: this model has {self.max_positions} positions")

    # ------------------------------------------------------------------ the pass
    def _forward(self, a: LatentPageAllocator, rows: int, ids, pos, row_seq, table, slots, runs, runs_host: np.ndarray, want, n_want: int, logits, logprobs=None,
                 nxt=None, advance: bool = False, history=None, graph: bool = False, tap=None) -> None:
        p = lambda t: None if t is None else t.data_ptr()  # noqa: E731
        slabs = (C.c_void_p * len(a.slabs))(*[s.data_ptr() if s.numel() else None for s in a.slabs])
        states = (C.c_void_p * len(a.slabs))(*[None if s is None else s.data_ptr() for s in a.states]) if self.recurrent else None
        b = _ffi.pie_stack_batch(rows, table.shape[0], table.shape[1], len(runs_host), n_want, int(advance), 0 if history is None else history.numel(), 0,
                                 p(ids), p(pos), p(row_seq), p(table), p(runs), runs_host.ctypes.data, p(want), p(logits), p(logprobs), p(nxt), p(history),
                                 C.cast(slabs, C.c_void_p), a.size(), p(tap), p(slots), None if states is None else C.cast(states, C.c_void_p),
                                 a.num_slots if self.recurrent else 0)
        _ffi.check(_ffi.base().pie_stack_forward(self._stack, C.byref(b), _ffi.PIE_STEP_GRAPH if graph else 0, _ffi.stream()))

    def _pass(self, entries: list, want: list[list[int]], tail: bool, tap=None):
        """entries: (token ids, sequence) -- ids a host array, or a device tensor of one token; want: places per entry.
        Returns (logits [n, V], logprobs, next) of the wanted rows, in the entries' order; the sequences advance.  The rows are laid out with the short
        runs first: the native pass serves those in the latent form and the long ones behind them with keys and values spelled out."""
        a = self._sequences([s for _, s in entries])
        for ids, s in entries:
            self._reserve(s, len(ids))
        S, lens = len(entries), np.asarray([len(i) for i, _ in entries], dtype=np.int32)
        order = np.argsort(lens, kind="stable")
        starts = np.empty(S, dtype=np.int32)
        starts[order] = np.concatenate([[0], np.cumsum(lens[order])[:-1]])
        M = int(lens.sum())
        width = max(len(s.pages) for _, s in entries)
        host = np.zeros(3 * M + S * width + 4 * S + S + M, dtype=np.int32)
        ids, pos, row_seq = host[:M], host[M:2 * M], host[2 * M:3 * M]
        table, runs = host[3 * M:3 * M + S * width].reshape(S, width), host[3 * M + S * width:3 * M + S * width + 4 * S].reshape(S, 4)
        on_device = []
        wanted: list[int] = []
        for i, (tok, s) in enumerate(entries):
            lo, hi = starts[i], starts[i] + lens[i]
            if isinstance(tok, torch.Tensor):
                on_device.append((lo, tok))
            else:
                ids[lo:hi] = tok
            pos[lo:hi] = np.arange(s.offset, s.offset + lens[i])
            row_seq[lo:hi] = i
            table[i, :len(s.pages)] = s.pages
            if self.recurrent:
                host[len(host) - M - S + i] = s.slot
            wanted += [int(lo) + int(k) for k in want[i]]
        for j, i in enumerate(order):
            runs[j] = (starts[i], lens[i], i, entries[i][1].offset)
        n_want = len(wanted)
        host[-M:][:n_want] = wanted
        dev = torch.from_numpy(host).to(self.device)
        for lo, tok in on_device:
            dev[lo:lo + 1].copy_(tok.reshape(-1))
        logits = torch.empty((n_want, self.vocab_size), dtype=torch.float32, device=self.device)
        logprobs = torch.empty_like(logits) if tail else None
        nxt = torch.empty(n_want, dtype=torch.int32, device=self.device) if tail else None
        o = 3 * M
        self._forward(a, M, dev[:M], dev[M:2 * M], dev[2 * M:o], dev[o:o + S * width].view(S, width), dev[-M - S:-M], dev[o + S * width:o + S * width + 4 * S], runs,
                      dev[-M:], n_want, logits, logprobs, nxt, tap=tap)
        for (_, s), n in zip(entries, lens):
            s.advance(int(n))
        return logits, logprobs, nxt

    def _portions(self, entries: list, want: list[list[int]], tail: bool):
        """_pass in pieces of at most MAX_ROWS rows."""
        if sum(len(t) for t, _ in entries) <= MAX_ROWS:
            return self._pass(entries, want, tail)
        self._sequences([s for _, s in entries])
        for t, s in entries:
            self._check_length(s, len(t))
        outs, batch, wants, room = [], [], [], MAX_ROWS

        def flush():
            nonlocal batch, wants, room
            if batch:
                outs.append(self._pass(batch, wants, tail))
            batch, wants, room = [], [], MAX_ROWS
        for (tok, s), w in zip(entries, want):
            at = 0
            while at < len(tok):
                n = min(room, len(tok) - at)
                batch.append((tok[at:at + n], s))
                wants.append([k - at for k in w if at <= k < at + n])
                at, room = at + n, room - n
                if room == 0:
                    flush()
        flush()
        return tuple(torch.cat(t) if t[0] is not None else None for t in zip(*outs))

    def step_portions(self, portions: list, want: list[list[int]]) -> torch.Tensor:
        """portions: (token ids, cache) per sequence -- a whole prompt, the next part of one, or one decoded token; all run as one batch behind what
        the caches hold.  want: per portion, the places among its tokens whose logits are returned: fp32 [total wanted, vocab]."""
        for (tok, _), w in zip(portions, want):
            if len(tok) == 0 or any(not 0 <= int(k) < len(tok) for k in w) or list(w) != sorted(set(w)):
                raise ValueError("a portion holds at least one token, and its wanted places are increasing places among them")
        return self._portions([(np.asarray(t, dtype=np.int32), self._sequence(c)) for t, c in portions], want, tail=False)[0]

    # ------------------------------------------------------------------ decode steps
    def _decode(self, tokens: torch.Tensor | None, seqs: list[PagedSequence], graph: bool, history=None) -> dict:
        """One token for each of the sequences from persistent buffers (per batch size), replayed as a captured graph.  tokens None: the ids the
        previous step of this batch left on the device."""
        a = self._sequences(seqs)
        B = len(seqs)
        for s in seqs:
            self._reserve(s, 1)
        mb = max(len(s.pages) for s in seqs)
        buf = self._bufs.pop(B, None)
        if buf is None or buf["table"].shape[1] < mb:
            width = max(mb, 2 * buf["table"].shape[1] if buf is not None else 4)
            i32 = dict(dtype=torch.int32, device=self.device)
            runs = np.stack([np.arange(B), np.ones(B), np.arange(B), np.zeros(B)], axis=1).astype(np.int32)
            buf = {"ids": torch.zeros(B, **i32), "pos": torch.zeros(B, **i32), "row_seq": torch.arange(B, **i32), "table": torch.zeros((B, width), **i32),
                   "runs_host": runs, "runs": torch.from_numpy(runs).to(self.device), "next": torch.empty(B, **i32),
                   "logits": torch.empty((B, self.vocab_size), dtype=torch.float32, device=self.device),
                   "logprobs": torch.empty((B, self.vocab_size), dtype=torch.float32, device=self.device), "slots": torch.zeros(B, **i32),
                   "pages": None, "held": None, "at": None}
            if tokens is None:
                raise RuntimeError("no previous step to continue from")
        while len(self._bufs) >= 4:
            self._bufs.pop(next(iter(self._bufs)))
        self._bufs[B] = buf
        pages = tuple(tuple(s.pages) for s in seqs)
        if buf["pages"] != pages:
            t = np.zeros(tuple(buf["table"].shape), dtype=np.int32)
            for i, s in enumerate(seqs):
                t[i, :len(s.pages)] = s.pages
            buf["table"].copy_(torch.from_numpy(t))
            buf["pages"] = pages
        if self.recurrent:
            held = [s.slot for s in seqs]
            if buf["held"] != held:
                buf["slots"].copy_(torch.tensor(held, dtype=torch.int32))
                buf["held"] = held
        at = [s.offset for s in seqs]
        if buf["at"] != at:
            buf["pos"].copy_(torch.tensor(at, dtype=torch.int32))
        if tokens is not None:
            buf["ids"].copy_(tokens.reshape(-1))
        self._forward(a, B, buf["ids"], buf["pos"], buf["row_seq"], buf["table"], buf["slots"], buf["runs"], buf["runs_host"], None, B, buf["logits"], buf["logprobs"],
                      buf["next"], advance=True, history=history, graph=graph)
        buf["at"] = [n + 1 for n in at]
        for s in seqs:
            s.advance(1)
        return buf

    def step(self, ids: torch.Tensor | None, cache: list[BaseCache], graph: bool = True):
        """Forwards `ids` [L] and returns (greedy token [1], logprobs [V], logits [V]) of the last position.  None feeds back the previous step's
        token, which is still on the device.  token stays valid; the other two until the next call."""
        seq = self._sequence(cache)
        L = 1 if ids is None else ids.numel()
        if L == 1:
            tok = None if ids is None else ids.reshape(-1).to(device=self.device, dtype=torch.int32)
            if ids is None and self._fed is not seq:
                raise RuntimeError("step(None) continues the sequence of the previous step")
            if tok is None and (1 not in self._bufs or self._bufs[1]["at"] != [seq.offset] or self._bufs[1]["table"].shape[1] * TOKEN_CAPACITY_PER_PAGE <= seq.offset):
                tok = self._last
            buf = self._decode(tok, [seq], graph, history=self.history)
            nxt, logprobs, logits = buf["next"], buf["logprobs"], buf["logits"]
            token = self.history[seq.offset:seq.offset + 1] if seq.offset < self.history.numel() else nxt.clone()
        else:
            host = ids.reshape(-1).to(torch.int32).cpu().numpy()
            logits, logprobs, nxt = self._portions([(host, seq)], [[L - 1]], tail=True)
            token = nxt
        self._fed, self._last = seq, token
        return token, logprobs[0], logits[0]

    _fed = _last = None

    def step_embeds(self, inputs_embeds, cache):
        raise NotImplementedError("a layer-stack model takes token ids (its experts or bigrams are chosen by them)")

    def step_batch(self, tokens: torch.Tensor, caches: list[list[BaseCache]], graph: bool = True):
        """One decode step of several sequences: (next tokens [B], logprobs [B, V], logits [B, V]), buffers valid until the next step of that size."""
        seqs = [self._sequence(c) for c in caches]
        tokens = tokens.to(device=self.device, dtype=torch.int32).reshape(-1)
        if tokens.numel() != len(seqs):
            raise ValueError("step_batch: one token per sequence")
        buf = self._decode(tokens, seqs, graph)
        self._fed = None
        return buf["next"], buf["logprobs"], buf["logits"]

    def prefill_batch(self, prompts: list, caches: list[list[BaseCache]]):
        """Several fresh prompts in one pass: (next tokens [S], logprobs, logits) of their last positions."""
        if any(c[0].offset != 0 for c in caches):
            raise ValueError("prefill_batch takes fresh caches")
        return self.step_mixed(None, [], prompts, caches)

    def step_mixed(self, tokens, decode_caches: list[list[BaseCache]], prompts: list, prompt_caches: list[list[BaseCache]]):
        """Decoding sequences and prompts (fresh, or continuing what their caches hold) in one pass; results as in step_batch, the decoding
        sequences first, then every prompt's last position."""
        entries = []
        if decode_caches:
            tokens = torch.as_tensor(tokens).to(device=self.device, dtype=torch.int32).reshape(-1)
            if tokens.numel() != len(decode_caches):
                raise ValueError("step_mixed: one token per decoding sequence")
            entries += [(tokens[i:i + 1], self._sequence(c)) for i, c in enumerate(decode_caches)]
        if any(len(p) == 0 for p in prompts) or len(prompts) != len(prompt_caches):
            raise ValueError("step_mixed: one non-empty prompt per cache")
        entries += [(np.asarray(p, dtype=np.int32).reshape(-1), self._sequence(c)) for p, c in zip(prompts, prompt_caches)]
        if not entries:
            raise ValueError("step_mixed: an empty batch")
        self._fed = None
        logits, logprobs, nxt = self._portions(entries, [[len(t) - 1] for t, _ in entries], tail=True)
        return nxt, logprobs, logits

    def __call__(self, inputs: torch.Tensor, mask=None, cache: list[BaseCache] | None = None, inputs_embeds=None) -> torch.Tensor:
        """inputs [1, L] -> logits [1, L, V] (fp32) behind what `cache` holds."""
        if inputs_embeds is not None:
            self.step_embeds(inputs_embeds, cache)
        if inputs.dim() != 2 or inputs.shape[0] != 1:
            raise ValueError("inputs must be [1, L]")
        if mask is not None and not (isinstance(mask, str) and mask == "causal"):
            raise NotImplementedError("a layer-stack model's layers carry their own masks")
        cache = self.make_cache() if cache is None else cache
        host = inputs.reshape(-1).to(torch.int32).cpu().numpy()
        return self._portions([(host, self._sequence(cache))], [list(range(len(host)))], tail=False)[0].unsqueeze(0)

    def layer_outputs(self, ids, cache: list[BaseCache] | None = None) -> torch.Tensor:
        """The residual stream behind every layer for one portion: fp32 [layers, L, width]."""
        host = np.asarray(ids, dtype=np.int32).reshape(-1)
        tap = torch.empty((len(self.layers), len(host), self.width), dtype=torch.float32, device=self.device)
        self._pass([(host, self._sequence(self.make_cache() if cache is None else cache))], [[]], tail=False, tap=tap)
        return tap

    def launches(self) -> int:
        """Kernel launches of the last pass that was not a graph replay."""
        return int(_ffi.base().pie_stack_launches(self._stack))


__all__ = ["Embedding", "LayerStackModel", "Norm", "interleave", "pack_linear", "pad", "pad_head_columns", "pad_head_rows", "up8", "yarn_frequencies"]
