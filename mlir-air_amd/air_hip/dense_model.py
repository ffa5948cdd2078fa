"""What the dense-weight models (kuvonex.py, sitirax.py) share: reading a checkpoint, the cache of one sequence, and the steps of
generation.CausalLM on top of two passes that a model provides:

  _one_token(cache, token, pos, pos_dev)   one token (device int32 [1]) through every layer -> what the tail reads
  _rows(cache, tokens, pos, trace)         many tokens -> the fp32 residual [M, width]

with `_head(pending, keys)` (fp32 logits of one position) and `_head_rows(res, rows)` (of some rows of a residual).
"""

import torch

from . import dense, generation, weights as wmod


def place(t, shape):
    """t in the corner of a zero tensor of `shape`."""
    if tuple(t.shape) == tuple(shape):
        return t
    out = torch.zeros(shape, dtype=t.dtype, device=t.device)
    out[tuple(slice(0, n) for n in t.shape)] = t
    return out


def checkpoint_reader(path):
    """tensor(name, shape) of a checkpoint directory; None in a shape stands for any length."""
    shards = wmod.SafetensorsDir(path)

    def tensor(name, shape):
        t = shards.tensor(name)
        if len(t.shape) != len(shape) or any(n is not None and n != m for n, m in zip(shape, t.shape)):
            raise ValueError(f"{name}: shape {tuple(t.shape)}, the configuration gives {tuple(shape)}")
        return t

    return tensor


class SequenceCache:
    """One sequence: the number of its tokens, and what a captured decode step keeps on the device.  Models add what their layers
    keep."""

    def __init__(self, model, capacity):
        self.capacity, self.pos = capacity, 0
        self.token = torch.zeros((1,), dtype=torch.int32, device=model.device)
        self.position = torch.zeros((1,), dtype=torch.int32, device=model.device)
        self.history = torch.zeros((capacity + 1,), dtype=torch.int32, device=model.device)
        self.graph = None

    def reset(self):
        self.pos = 0


class DenseModel(generation.CausalLM):
    max_portion = None       # most tokens that go through the layers at once (None: any number)

    @classmethod
    def load(cls, path, config_json, dtype=torch.bfloat16, device="cuda"):
        return cls(cls.config_class.from_json(config_json), checkpoint_reader(path), dtype, device)

    def _captured_decode(self):
        """Whether a decode step can run with the position on the device."""
        return True

    def _ids(self, tokens):
        if isinstance(tokens, torch.Tensor):   # already on the device: the caller answers for the range
            return tokens.to(device=self.device, dtype=torch.int32).contiguous()
        tokens = [int(t) for t in tokens]
        if not tokens or min(tokens) < 0 or max(tokens) >= self.vocab:
            raise ValueError(f"token ids must lie in 0 .. {self.vocab - 1}")
        return torch.tensor(tokens, dtype=torch.int32, device=self.device)

    def _advance(self, cache, n):
        if cache.pos + n > cache.capacity:
            raise ValueError(f"the sequence needs {cache.pos + n} tokens, its cache holds {cache.capacity}")
        pos, cache.pos = cache.pos, cache.pos + n
        return pos

    def _portions(self, n):
        size = self.max_portion or n
        return [(i, min(i + size, n)) for i in range(0, n, size)]

    def _tail(self, pending):
        keys = dense.new_keys(self.head)
        logits = self._head(pending, keys)
        best = torch.empty((1,), dtype=torch.int32, device=self.device)
        dense.argmax(keys, best)
        return logits[:self.vocab], best

    # -- generation.CausalLM ---------------------------------------------------------------
    def step(self, cache, tokens, want, trace=None):
        ids = self._ids(tokens)
        pos = self._advance(cache, len(ids))
        none = torch.empty((0, self.vocab), device=self.device)
        if len(ids) == 1 and trace is None:
            pending = self._one_token(cache, ids, pos)
            return self._head(pending)[:self.vocab].reshape(1, -1).expand(len(want), -1) if want else none
        order, logits = [], []
        for a, b in self._portions(len(ids)):
            res = self._rows(cache, ids[a:b], pos + a, trace)
            here = [i for i, w in enumerate(want) if a <= w < b]
            if here:
                order += here
                rows = torch.tensor([want[i] - a for i in here], dtype=torch.int32, device=self.device)
                logits.append(self._head_rows(res, rows)[:, :self.vocab])
        if not order:
            return none
        out = logits[0] if len(logits) == 1 else torch.cat(logits)
        return out if order == sorted(order) else out[torch.tensor(sorted(range(len(order)), key=order.__getitem__), device=self.device)]

    def prefill(self, cache, tokens):
        ids = self._ids(tokens)
        pos = self._advance(cache, len(ids))
        if len(ids) == 1:
            return self._tail(self._one_token(cache, ids, pos))
        for a, b in self._portions(len(ids)):
            res = self._rows(cache, ids[a:b], pos + a)
        return self._tail(self._pending(res[-1].contiguous()))

    def decode_token(self, cache, token):
        pos = self._advance(cache, 1)
        return self._tail(self._one_token(cache, self._ids([token]), pos))

    def _greedy_step(self, cache):
        """The token and position kept on the device -> the next token and position there."""
        pending = self._one_token(cache, cache.token, 0, cache.position)
        keys = dense.new_keys(self.head)
        self._head(pending, keys)
        dense.argmax(keys, cache.token, cache.position, cache.history)

    def decode_greedy(self, cache, first, n_tokens):
        """The step is captured as a HIP graph the first time a cache decodes (token and position live on the device)
        and replayed per token; inside a caller's capture the launches are recorded one by one."""
        start = self._advance(cache, n_tokens)
        if not self._captured_decode():
            return self._decode_eagerly(cache, first, start, n_tokens)
        capturing = torch.cuda.is_current_stream_capturing()
        cache.token.copy_(first.to(torch.int32).reshape(1))
        cache.position.fill_(start)
        if capturing:
            for _ in range(n_tokens):
                self._greedy_step(cache)
        elif n_tokens > 0:
            if cache.graph is None:
                self._greedy_step(cache)    # the first token runs as it is: nothing is set up for the first time in the capture
                n_tokens -= 1
                torch.cuda.synchronize()
                cache.graph = torch.cuda.CUDAGraph()
                with torch.cuda.graph(cache.graph):
                    self._greedy_step(cache)
            for _ in range(n_tokens):
                cache.graph.replay()
        return cache.history[start + 1:cache.pos + 1].clone()

    def _decode_eagerly(self, cache, first, start, n_tokens):
        out, tok = [], first.to(torch.int32).reshape(1)
        for i in range(n_tokens):
            _, tok = self._tail(self._one_token(cache, tok, start + i))
            out.append(tok)
        return torch.cat(out) if out else torch.empty((0,), dtype=torch.int32, device=self.device)

    def check_health(self):
        torch.cuda.synchronize()
