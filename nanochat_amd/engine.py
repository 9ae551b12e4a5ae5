"""KV cache, next-token sampler and the batched generation loop, API-compatible with nanochat/engine.py
(KVCache :82-137, sample_next_token :140-156, Engine :169-299, calculator :25-79).

Device work (model forward, sampling on GPU logits) goes to the HIP kernels; this file is host logic:
cache bookkeeping, the per-row tool-use state machine and the streaming generator protocol.
"""
import ctypes
import signal
import warnings
from collections import deque
from contextlib import contextmanager

import torch
import torch.nn.functional as F

from . import ops
from .common import COMPUTE_DTYPE

# ------------------------------------------------------------------------------------------------
# Calculator tool (engine.py:25-79): evaluates the text between <|python_start|> and <|python_end|>.
_MATH_CHARS = set("0123456789*+-/.() ")
_TEXT_CHARS = set("abcdefghijklmnopqrstuvwxyzABCDEFGHIJKLMNOPQRSTUVWXYZ0123456789'\"()._ ")
_BANNED = ("__", "import", "exec", "eval", "compile", "open", "file", "input", "raw_input", "globals", "locals",
           "vars", "dir", "getattr", "setattr", "delattr", "hasattr")


class _CalcTimeout(Exception):
    pass


@contextmanager
def _alarm(seconds, what):
    def on_alarm(signum, frame):
        raise _CalcTimeout(f"'{what}': timed out after {seconds} seconds")
    signal.signal(signal.SIGALRM, on_alarm)
    signal.alarm(seconds)
    try:
        yield
    finally:
        signal.alarm(0)


def eval_with_timeout(formula, max_time=3):
    """eval() with empty builtins under a SIGALRM limit; None on any failure."""
    try:
        with _alarm(max_time, formula), warnings.catch_warnings():
            warnings.simplefilter("ignore", SyntaxWarning)
            return eval(formula, {"__builtins__": {}}, {})
    except Exception:
        return None


def use_calculator(expr):
    """Arithmetic over + - * / ( ) (no **), or a quoted-string .count(...) expression; else None."""
    expr = expr.replace(",", "")
    if set(expr) <= _MATH_CHARS:
        return None if "**" in expr else eval_with_timeout(expr)
    if not set(expr) <= _TEXT_CHARS:
        return None
    lowered = expr.lower()
    if any(word in lowered for word in _BANNED):
        return None
    if ".count(" not in expr:
        return None
    return eval_with_timeout(expr)


# ------------------------------------------------------------------------------------------------
class SequenceCache:
    """Positions of the rows of a cache: per-row lengths in an int32 device tensor, with a host-side copy so that get_pos() does not
    have to read the device tensor back every decode step.  What the rows hold is the subclass's: keys and values (KVCache), or
    token rows and recurrent states (StackCache).  The Engine uses: get_pos, advance / note_advanced (by the model), mark and rewind."""

    def __init__(self, batch_size, seq_len, device):
        self.batch_size = batch_size
        self.max_seq_len = seq_len
        self.cache_seqlens = torch.zeros(batch_size, dtype=torch.int32, device=device)
        self._pos0 = 0          # host mirror of cache_seqlens[0]
        self._pos_max = 0       # host mirror of cache_seqlens.max()

    def get_pos(self):
        return self._pos0

    def advance(self, num_tokens):
        self.cache_seqlens += num_tokens
        self._moved(num_tokens)

    def note_advanced(self, num_tokens):
        """The forward call advanced `cache_seqlens` on the device itself (the `advance` field of its cache descriptor): only the host
        side follows."""
        self._moved(num_tokens)

    def _moved(self, num_tokens):
        self._pos0 += num_tokens
        self._pos_max += num_tokens

    def mark(self):
        """What rewind() needs to take back the forward that follows."""
        return None


class KVCache(SequenceCache):
    """Pre-allocated (n_layers, B, T, H, D) key and value tensors in FA3 layout, per-row lengths in an
    int32 tensor, and the previous token's normalised embedding for the smear gate (engine.py:82-137).

    The host-side copy of the position is exact as long as positions change only through advance/reset/prefill
    (or set_seqlens for ragged batches, where it tracks row 0 like the reference's get_pos)."""

    def __init__(self, batch_size, num_heads, seq_len, head_dim, num_layers, device, dtype, prefill_from=None, share_prompt_reads=False):
        """prefill_from (not in the reference's signature): another cache whose tokens this one starts with, i.e.
        KVCache(...) followed by .prefill(prefill_from) in one step.  On the GPU the tensors then never get the zero fill that the
        copy would overwrite anyway (at d26 / 64 rows / 1792 prompt tokens that fill is 20 of the 22.7 GB, 4 ms of the time to the
        first token): only the positions past the prompt are cleared, and the end state is the same.

        share_prompt_reads (not in the reference's signature, off by default): after a prefill from a batch-1 cache every row holds a
        copy of the same prompt.  With this set the cache remembers how long that shared start is (`shared_prefix_len`) and a one-token
        forward reads it once for all rows in the layers that see most of it, instead of once per row; the tensors keep the reference's
        layout and contents.  The promise that goes with it: nobody writes into positions [0, shared_prefix_len) of k_cache / v_cache
        by hand (set shared_prefix_len = 0 first)."""
        super().__init__(batch_size, seq_len, device)
        self.n_layers = num_layers
        self.n_heads = num_heads
        self.head_dim = head_dim
        shape = (num_layers, batch_size, seq_len, num_heads, head_dim)
        lazy = prefill_from is not None and torch.device(device).type == "cuda"
        alloc = torch.empty if lazy else torch.zeros
        self.k_cache = alloc(shape, device=device, dtype=dtype)
        self.v_cache = alloc(shape, device=device, dtype=dtype)
        self.prev_embedding = None
        self.share_prompt_reads = bool(share_prompt_reads)
        self.shared_prefix_len = 0      # positions [0, this) hold the same bytes in every row (set by prefill from a batch-1 cache)
        if prefill_from is not None:
            if lazy:
                n = prefill_from.get_pos()
                assert seq_len >= prefill_from.max_seq_len >= n
                self.k_cache[:, :, n:].zero_()
                self.v_cache[:, :, n:].zero_()
            self.prefill(prefill_from)

    def reset(self):
        self.cache_seqlens.zero_()
        self.prev_embedding = None
        self._pos0 = self._pos_max = 0
        self.shared_prefix_len = 0

    def get_layer_cache(self, layer_idx):
        return self.k_cache[layer_idx], self.v_cache[layer_idx]

    def mark(self):
        return self.prev_embedding

    def rewind(self, num_tokens, prev_embedding):
        """Take back the last advance (the appended rows stay in the tensors and are overwritten by the next
        append at the same positions); `prev_embedding` is the smear state from before that forward."""
        assert 0 < num_tokens <= self._pos0
        self.cache_seqlens -= num_tokens
        self._pos0 -= num_tokens
        self._pos_max -= num_tokens
        self.prev_embedding = prev_embedding
        if self._pos0 < self.shared_prefix_len:         # the next append would land inside the shared start
            self.shared_prefix_len = 0

    def set_seqlens(self, seqlens):
        """Ragged rows: install per-row lengths (host list or tensor)."""
        t = torch.as_tensor(seqlens, dtype=torch.int32)
        assert t.shape == (self.batch_size,)
        self._pos0, self._pos_max = int(t[0]), int(t.max())
        assert 0 <= int(t.min()) and self._pos_max <= self.max_seq_len
        self.cache_seqlens.copy_(t)
        self.shared_prefix_len = 0

    def prefill(self, other):
        """Copy another cache's first pos tokens into every row of this one (engine.py:123-137)."""
        assert self.get_pos() == 0, "Cannot prefill a non-empty KV cache"
        assert self.n_layers == other.n_layers and self.n_heads == other.n_heads and self.head_dim == other.head_dim
        assert self.max_seq_len >= other.max_seq_len
        n = other.get_pos()
        if self.k_cache.is_cuda:
            assert other.batch_size in (1, self.batch_size)
            ops.kv_cache_prefill(self.k_cache, other.k_cache, n)
            ops.kv_cache_prefill(self.v_cache, other.v_cache, n)
        else:           # host-side caches (the engine's own logic under test with a mock model)
            self.k_cache[:, :, :n, :, :] = other.k_cache[:, :, :n, :, :]
            self.v_cache[:, :, :n, :, :] = other.v_cache[:, :, :n, :, :]
        self.cache_seqlens.fill_(n)
        self._pos0 = self._pos_max = n
        self.shared_prefix_len = n if (other.batch_size == 1 and self.batch_size > 1) else 0
        if other.prev_embedding is not None:
            self.prev_embedding = other.prev_embedding.expand(self.batch_size, -1, -1).clone()


class StackCache(SequenceCache):
    """Cache of a layer stack (nanochat_amd/stack.py): for every run of an attention mixer a row per token (latents, or
    keys and values), for every run of a recurrent mixer one fp32 state per sequence.  A layer that runs several times has slots for each
    of its runs.

    `rows[slot]` [B, seq_len, row width]; `states[i][slot]` [B, ...], two buffers: a forward reads one and writes the other, so a forward can be taken back.  A row at position 0 does not read its state: a slot of the batch is given back by
    setting its position to zero."""

    def __init__(self, row_widths, state_shapes, dtype, batch_size, seq_len, device, prefill_from=None):
        super().__init__(batch_size, seq_len, device)
        self.dtype = dtype
        # (zeros: the positions past a row's end enter products with weight zero, and must be finite there)
        self.rows = [torch.zeros(batch_size, seq_len, w, device=device, dtype=dtype) for w in row_widths]
        self.states = [[torch.zeros(batch_size, *s, device=device, dtype=torch.float32) for s in state_shapes] for _ in range(2)]
        self._pointers = None
        self._current = 0                          # which of the two state buffers holds the states
        self._host_pos = [0] * batch_size
        self._last_tokens = 0                      # tokens of the last forward, which is the one rewind() can take back
        if prefill_from is not None:
            self.prefill(prefill_from)

    def _positions_changed(self):
        self._pos0, self._pos_max = self._host_pos[0], max(self._host_pos)
        self._last_tokens = 0

    def reset(self):
        self.reset_rows(range(self.batch_size))

    def reset_rows(self, rows):
        """Give rows of the batch back: their next token is the first of a new sequence."""
        for r in rows:
            self.cache_seqlens[r] = 0
            self._host_pos[r] = 0
        self._positions_changed()

    def state_buffers(self):
        """(states to read, states to write) of the next forward."""
        return self.states[self._current], self.states[self._current ^ 1]

    def pointers(self):
        """Arrays of device pointers: token rows, states to read, states to write (the tensors of a cache never move)."""
        if self._pointers is None:
            lat, a, b = ((ctypes.c_void_p * max(1, len(ts)))(*(t.data_ptr() for t in ts)) for ts in (self.rows, *self.states))
            self._pointers = ((lat, a, b), (lat, b, a))
        return self._pointers[self._current]

    def _moved(self, num_tokens):
        super()._moved(num_tokens)
        self._host_pos = [p + num_tokens for p in self._host_pos]
        self._current ^= 1
        self._last_tokens = num_tokens

    def rewind(self, num_tokens, mark=None):
        """Take back the last forward, which brought `num_tokens` tokens (their rows are overwritten by the next ones)."""
        assert 0 < num_tokens == self._last_tokens, "only the last forward can be taken back"
        self.cache_seqlens -= num_tokens
        self._host_pos = [p - num_tokens for p in self._host_pos]
        self._positions_changed()
        self._current ^= 1

    def load_row(self, row, other, other_row=0):
        """Copy one sequence out of another cache of the same model into row `row` of this one."""
        self._copy(other, other_row, 1, row, 1)
        self.cache_seqlens[row] = other._host_pos[other_row]
        self._host_pos[row] = other._host_pos[other_row]
        self._positions_changed()

    def prefill(self, other):
        """Copy another cache's tokens and states into every row of this one (row by row, or its one row into all)."""
        assert self._pos_max == 0, "Cannot prefill a non-empty cache"
        assert other.batch_size in (1, self.batch_size)
        self._copy(other, 0, other.batch_size, 0, self.batch_size)
        self._host_pos = list(other._host_pos) if other.batch_size == self.batch_size else other._host_pos * self.batch_size
        self.cache_seqlens.copy_(torch.tensor(self._host_pos, dtype=torch.int32))
        self._positions_changed()

    def _copy(self, other, src_row, src_rows, dst_row, dst_rows):
        n = other._pos_max
        assert n <= self.max_seq_len and self.dtype == other.dtype
        assert [t.shape[2] for t in self.rows] == [t.shape[2] for t in other.rows]
        for src, dst in zip(other.rows, self.rows):
            ops.stack_cache_copy(src[src_row:src_row + src_rows], dst[dst_row:dst_row + dst_rows], n)
        for src, dst in zip(other.state_buffers()[0], self.state_buffers()[0]):
            ops.stack_cache_copy(src[src_row:src_row + src_rows], dst[dst_row:dst_row + dst_rows], src.shape[1])


# ------------------------------------------------------------------------------------------------
@torch.inference_mode()
def sample_next_token(logits, rng, temperature=1.0, top_k=None):
    """(B, vocab) logits -> (B, 1) token ids (engine.py:140-156).

    GPU logits: the HIP sampler; the Exp(1) variates of the multinomial draw come from `rng`.
    CPU logits (host-side tests with a mock model): the same steps in torch."""
    assert temperature >= 0.0, "temperature must be non-negative"
    if logits.is_cuda:
        logits = logits.float()
        if temperature == 0.0:
            return ops.sample(logits, 0.0, None, None)
        B, V = logits.shape
        k = min(top_k, V) if (top_k is not None and top_k > 0) else V
        noise = torch.empty(B, k, dtype=torch.float32, device=logits.device).exponential_(1.0, generator=rng)
        return ops.sample(logits, temperature, top_k, noise)
    if temperature == 0.0:
        return torch.argmax(logits, dim=-1, keepdim=True)
    if top_k is not None and top_k > 0:
        vals, idx = torch.topk(logits, min(top_k, logits.size(-1)), dim=-1)
        choice = torch.multinomial(F.softmax(vals / temperature, dim=-1), num_samples=1, generator=rng)
        return idx.gather(1, choice)
    return torch.multinomial(F.softmax(logits / temperature, dim=-1), num_samples=1, generator=rng)


# ------------------------------------------------------------------------------------------------
class RowState:
    """Generation state of one batch row (engine.py:160-167)."""

    def __init__(self, current_tokens=None):
        self.current_tokens = current_tokens or []
        self.forced_tokens = deque()
        self.in_python_block = False
        self.python_expr_tokens = []
        self.completed = False


class _Specials:
    def __init__(self, tokenizer):
        self.python_start = tokenizer.encode_special("<|python_start|>")
        self.python_end = tokenizer.encode_special("<|python_end|>")
        self.output_start = tokenizer.encode_special("<|output_start|>")
        self.output_end = tokenizer.encode_special("<|output_end|>")
        self.assistant_end = tokenizer.encode_special("<|assistant_end|>")
        self.bos = tokenizer.get_bos_token_id()


class Engine:
    def __init__(self, model, tokenizer):
        self.model = model
        self.tokenizer = tokenizer

    def _step_row(self, state, sampled, sp):
        """Pick the row's next token (forced beats sampled), update the tool-use machine.
        Returns (token, mask) with mask 0 for forced and 1 for sampled (engine.py:238-267)."""
        forced = len(state.forced_tokens) > 0
        token = state.forced_tokens.popleft() if forced else sampled
        state.current_tokens.append(token)
        if token == sp.assistant_end or token == sp.bos:
            state.completed = True
        if token == sp.python_start:
            state.in_python_block = True
            state.python_expr_tokens = []
        elif token == sp.python_end and state.in_python_block:
            state.in_python_block = False
            if state.python_expr_tokens:
                result = use_calculator(self.tokenizer.decode(state.python_expr_tokens))
                if result is not None:
                    state.forced_tokens.append(sp.output_start)
                    state.forced_tokens.extend(self.tokenizer.encode(str(result)))
                    state.forced_tokens.append(sp.output_end)
            state.python_expr_tokens = []
        elif state.in_python_block:
            state.python_expr_tokens.append(token)
        return token, (0 if forced else 1)

    def _new_cache(self, batch_size, seq_len, prefill_from=None, share_prompt_reads=False):
        """A cache of the model's own kind (model.new_cache), or the KV cache that its configuration describes."""
        make = getattr(self.model, "new_cache", None)
        if make is not None:
            return make(batch_size, seq_len, prefill_from=prefill_from, share_prompt_reads=share_prompt_reads)
        cfg, device = self.model.config, self.model.get_device()
        dtype = torch.bfloat16 if torch.device(device).type == "cuda" else COMPUTE_DTYPE
        return KVCache(batch_size=batch_size, num_heads=cfg.n_kv_head, seq_len=seq_len, head_dim=cfg.n_embd // cfg.n_head, num_layers=cfg.n_layer,
                       device=device, dtype=dtype, prefill_from=prefill_from, share_prompt_reads=share_prompt_reads)

    def _last_logits(self, ids, kv_cache):
        fast = getattr(self.model, "forward_last", None)
        if fast is not None:
            return fast(ids, kv_cache=kv_cache)
        return self.model.forward(ids, kv_cache=kv_cache)[:, -1, :]

    @torch.inference_mode()
    def generate(self, tokens, num_samples=1, max_tokens=None, temperature=1.0, top_k=None, seed=42, share_prompt_reads=False, prefill_chunk=None):
        """One batch-1 prefill, cache replicated to num_samples rows, then streamed decoding.
        Yields (token_column, token_masks) per step (engine.py:175-275).

        share_prompt_reads (not in the reference's signature, off by default): every row's cache starts with a copy of the same
        prompt; with this set, the decode steps read that prompt once for all rows in the full-context layers (see KVCache).

        prefill_chunk (not in the reference's signature): the prompt goes through the model in portions of at most this many tokens
        (bounds the workspace of a long prompt); None: in one piece."""
        assert isinstance(tokens, list) and isinstance(tokens[0], int), "expecting list of ints"
        device = self.model.get_device()
        rng = torch.Generator(device=device)
        rng.manual_seed(seed)
        sp = _Specials(self.tokenizer)

        kv_prefill = self._new_cache(1, len(tokens))
        portion = len(tokens) if prefill_chunk is None else max(1, prefill_chunk)
        for start in range(0, len(tokens), portion):
            ids = torch.tensor([tokens[start:start + portion]], dtype=torch.long, device=device)
            logits = self._last_logits(ids, kv_prefill)
        logits = logits.expand(num_samples, -1)

        hint = (len(tokens) + max_tokens) if max_tokens is not None else max(self.model.config.sequence_len, len(tokens) + 1)
        kv_decode = self._new_cache(num_samples, hint, prefill_from=kv_prefill, share_prompt_reads=share_prompt_reads)
        del kv_prefill

        rows = [RowState(tokens.copy()) for _ in range(num_samples)]
        produced = 0
        # On the GPU the next forward is enqueued on the sampled ids before the host has seen them: the ids travel to a
        # pinned buffer by an async copy placed ahead of that forward, and the tool-use state machine runs while the
        # GPU computes.  If the machine then forces a different token for some row, the step is taken back (positions
        # and smear state) and redone with the forced column -- the outputs are those of the plain loop.
        ahead = torch.device(device).type == "cuda" and hasattr(self.model, "forward_last")
        if ahead:
            host_ids = torch.empty(num_samples, dtype=torch.long, pin_memory=True)
            ids_ready = torch.cuda.Event()
        while True:
            if max_tokens is not None and produced >= max_tokens:
                break
            if all(r.completed for r in rows):
                break
            sampled_dev = sample_next_token(logits, rng, temperature, top_k)
            # (not in front of the first token: the caller gets it as soon as it is sampled, as in the reference's loop, where the
            # time to the first token ends before the first decode forward)
            run_ahead = ahead and produced > 0 and not (max_tokens is not None and produced + 1 >= max_tokens)
            if run_ahead:
                # (on the launch stream: handing this copy to a stream of its own costs 90 us per step -- with a second queue
                # active every one of the step's ~190 launches starts ~0.5 us later)
                host_ids.copy_(sampled_dev[:, 0], non_blocking=True)
                ids_ready.record()
                before = kv_decode.mark()
                logits_ahead = self._last_logits(sampled_dev, kv_decode)
                ids_ready.synchronize()
                sampled = host_ids.tolist()
            else:
                sampled = sampled_dev[:, 0].tolist()
            column, masks = [], []
            for r, s in zip(rows, sampled):
                tok, mask = self._step_row(r, s, sp)
                column.append(tok)
                masks.append(mask)
            yield column, masks
            produced += 1
            if run_ahead and column == sampled:
                logits = logits_ahead
                continue
            if run_ahead:
                kv_decode.rewind(1, before)
            # forced tokens come from the tokenizer, not from the sampler: refuse what the embedding table does not hold
            rows_in_table = getattr(self.model, "padded_vocab_size", None)
            if rows_in_table is not None and not all(0 <= t < rows_in_table for t in column):
                raise IndexError(f"token id out of range for an embedding table of {rows_in_table} rows: {column}")
            ids = torch.tensor(column, dtype=torch.long, device=device).unsqueeze(1)
            logits = self._last_logits(ids, kv_decode)

    def generate_batch(self, tokens, num_samples=1, **kwargs):
        """Drain generate(); returns (sequences, masks) without terminal tokens (engine.py:277-299)."""
        sp = _Specials(self.tokenizer)
        results = [tokens.copy() for _ in range(num_samples)]
        masks = [[0] * len(tokens) for _ in range(num_samples)]
        done = [False] * num_samples
        for column, column_masks in self.generate(tokens, num_samples, **kwargs):
            for i, (tok, mask) in enumerate(zip(column, column_masks)):
                if done[i]:
                    continue
                if tok == sp.assistant_end or tok == sp.bos:
                    done[i] = True
                else:
                    results[i].append(tok)
                    masks[i].append(mask)
            if all(done):
                break
        return results, masks
