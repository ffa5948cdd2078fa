"""The token loop shared by every model: prompt pass, greedy decode, and the bookkeeping of caches between requests.

`generate` is the loop of the reference's `generate`
(programming_examples/llms/llama32_1b_int4/llama32_1b_int4_inference.py:494-575) with the model behind an interface:
the int4 Llama (decode.LlamaModel) and the dense-weight models (kuvonex.KuvonexModel, sitirax.SitiraxModel) all run through it.
"""


class UnsupportedDtype(ValueError):
    """The model has no kernels for the element type asked for."""


class CausalLM:
    """What the token loop needs from a model.  A cache holds one sequence (`pos` tokens of at most `capacity`) and is
    reused after `reset()`."""

    vocab = None
    device = None

    def new_cache(self, max_tokens):
        raise NotImplementedError

    def step(self, cache, tokens, want):
        """Run the next tokens (a list of ints) of the cache's sequence; fp32 logits [len(want), vocab] at the places
        `want` among them."""
        raise NotImplementedError

    def prefill(self, cache, tokens):
        """Run a prompt (ints, or ids on the device); (fp32 logits [vocab] of its last position, greedy next token as a device int32 [1])."""
        raise NotImplementedError

    def decode_token(self, cache, token):
        """Run one token (an int); the same pair for it."""
        raise NotImplementedError

    def decode_greedy(self, cache, first, n_tokens):
        """Greedy decode on the device from the token `first` (device int32 [1]): n_tokens ids, device int32."""
        raise NotImplementedError

    def check_health(self):
        """Raise if a launch since the last check left an invalid result; synchronises."""


class CachePool:
    """Caches of live requests, by request id; a finished request's cache serves a later one."""

    def __init__(self, model, max_tokens):
        self.model, self.max_tokens = model, max_tokens
        self.live, self.free = {}, []

    def get(self, request):
        if request not in self.live:
            cache = self.free.pop() if self.free else self.model.new_cache(self.max_tokens)
            cache.reset()
            self.live[request] = cache
        return self.live[request]

    def end(self, request):
        cache = self.live.pop(request, None)
        if cache is not None:
            self.free.append(cache)


def generate(model, prompt_tokens, n_tokens=10, eos_token_ids=(), on_token=None, cache=None):
    """[First token predicted by the prompt pass] + the tokens decoded after it, at most n_tokens of them, ending with
    the first end-of-sequence id if one is produced.

    Without `on_token` the whole decode loop runs on the device and the ids come back once; tokens after an
    end-of-sequence id are computed and dropped.  With `on_token(token_id)` every token is brought to the host as it is
    produced and the loop stops at an end-of-sequence id.  `cache`: one of model.new_cache to use (from its start)."""
    prompt = [int(t) for t in prompt_tokens]
    if not prompt:
        raise ValueError("generate needs at least one prompt token")
    if cache is None:
        cache = model.new_cache(len(prompt) + n_tokens)
    cache.reset()
    _, first = model.prefill(cache, prompt)
    eos = set(int(t) for t in eos_token_ids)
    if on_token is None:
        rest = model.decode_greedy(cache, first, n_tokens) if n_tokens > 0 else None
        model.check_health()
        out = [int(first.item())] + ([int(t) for t in rest.cpu().tolist()] if rest is not None else [])
        for i in range(1, len(out)):
            if out[i] in eos:
                return out[:i + 1]
        return out
    tok = int(first.item())
    out = [tok]
    on_token(tok)
    for _ in range(n_tokens):
        _, best = model.decode_token(cache, tok)
        model.check_health()
        tok = int(best.item())
        out.append(tok)
        on_token(tok)
        if tok in eos:
            break
    return out
