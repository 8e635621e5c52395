"""The token table, read at the bottom of the model (gather) and, tied, at the top (head)."""

from __future__ import annotations

from ..ops import kernels
from ..weights.spec import MATRIX, TABLE, Normal, TensorSpec
from .base import Part, PositionEncoding, StateNeed


class TokenEmbedding(Part):
    """``scale`` multiplies the token rows (in 32-bit, as they are gathered). ``tensor_name``: the table's name behind the
    part's prefix ("" where the part's own name is the tensor's)."""

    def __init__(self, vocab_size: int, width: int, scale: float = 1.0, tensor_name: str = "weight", std: float = 0.02):
        self.vocab_size, self.width, self.scale = vocab_size, width, float(scale)
        self._tensor_name, self._std = tensor_name, std
        self.weight = None

    def tensor_specs(self):
        return {self._tensor_name: TensorSpec((self.vocab_size, self.width), TABLE, Normal(self._std))}

    def bind(self, tensors):
        self.weight = tensors[self._tensor_name]

    def state_need(self) -> StateNeed | None:
        """What the embedding keeps of a sequence from step to step (nothing: a row is a function of its token and position)."""
        return None

    def forward(self, tokens, positions, position_encoding: PositionEncoding | None, token_sources=None, token_slots=None, batch=None, state=None):
        """[rows, width] float32: token rows, with the position rows added when the encoding
        is one that enters at the embedding (a table ``weight`` [positions, width]); an encoding
        of stage "mixer", or none, leaves the token rows as they are. ``token_sources`` /
        ``token_slots``: rows whose token is still on the device, in the slot the sampler left it
        in (kernels.embed). ``batch`` / ``state``: the step's batch and the slots of ``state_need``, for an embedding that keeps state."""
        table = position_encoding.weight if position_encoding is not None and position_encoding.stage == "embedding" else None
        return kernels.embed(tokens, positions, self.weight, table, token_sources=token_sources, token_slots=token_slots, scale=self.scale)


class PairEmbedding(TokenEmbedding):
    """A token's row plus a row of a second table [buckets + 1, width] picked by the token and the one before it in its sequence: row
    (previous * mul_previous + token * mul_current) mod buckets, and the last row for a sequence's first token. The previous token of
    a portion's first row is part of the sequence's state: one integer a state slot, read and moved on to the portion's last token
    inside the gather, also where that token is still on the device. ``pair_name``: the second table's name behind the part's prefix."""

    def __init__(self, vocab_size: int, width: int, *, buckets: int, mul_previous: int, mul_current: int, scale: float = 1.0,
                 tensor_name: str = "weight", pair_name: str = "pairs", std: float = 0.02):
        super().__init__(vocab_size, width, scale=scale, tensor_name=tensor_name, std=std)
        self.buckets, self.mul_previous, self.mul_current = buckets, mul_previous, mul_current
        self._pair_name = pair_name
        self.pairs = None

    def tensor_specs(self):
        return {**super().tensor_specs(), self._pair_name: TensorSpec((self.buckets + 1, self.width), TABLE, Normal(self._std))}

    def bind(self, tensors):
        super().bind(tensors)
        self.pairs = tensors[self._pair_name]

    def state_need(self):
        import torch

        return StateNeed((), torch.int32)

    def forward(self, tokens, positions, position_encoding: PositionEncoding | None, token_sources=None, token_slots=None, batch=None, state=None):
        if position_encoding is not None and position_encoding.stage == "embedding":
            raise ValueError("no position rows are added to token pairs")
        pairs = kernels.TokenPairs(self.pairs, self.mul_previous, self.mul_current, batch.token_request, batch.q_starts, batch.state_slots, state)
        return kernels.embed(tokens, positions, self.weight, None, token_sources=token_sources, token_slots=token_slots, scale=self.scale, pairs=pairs)


class TiedHead(Part):
    """logits = x . wte^T, no bias, no tensor of its own (engine/src/gpt2.c:244-256)."""

    def __init__(self, embedding: TokenEmbedding):
        self.embedding = embedding

    def forward(self, x):
        import torch

        return kernels.linear(x, self.embedding.weight, out_dtype=torch.float32)

    def forward_best(self, x):
        """For a step that decodes greedily: instead of the logits, per row the best (logit, token) of each of a few
        hundred disjoint parts of the vocabulary (kernels.linear_best), among which ``kernels.choose`` finds the row's
        argmax; None where that kernel does not take the sizes (the caller then takes the logits). A head without this
        method is asked for its logits."""
        if not kernels.best_per_row(x.shape[0], self.embedding.weight, x.dtype):
            return None
        return kernels.linear_best(x, self.embedding.weight)


class LinearHead(Part):
    """logits = x . W^T with a matrix of its own, [vocab, width], no bias. ``softcap``: a logit z then counts as softcap tanh(z / softcap)."""

    def __init__(self, vocab_size: int, width: int, tensor_name: str = "weight", softcap: float | None = None):
        if softcap is not None and not softcap > 0:
            raise ValueError(f"the cap must be positive, not {softcap}")
        self.vocab_size, self.width, self.softcap = vocab_size, width, softcap
        self._tensor_name = tensor_name
        self.weight = None

    def tensor_specs(self):
        return {self._tensor_name: TensorSpec((self.vocab_size, self.width), MATRIX, Normal(self.width ** -0.5))}

    def bind(self, tensors):
        self.weight = tensors[self._tensor_name]

    def forward(self, x):
        import torch

        logits = kernels.linear(x, self.weight, out_dtype=torch.float32)
        return logits if self.softcap is None else kernels.soft_cap(logits, self.softcap, out=logits)

    def forward_best(self, x):
        """See TiedHead.forward_best. (A cap does not change which logit is the largest: the pairs hold what goes into it.)"""
        if not kernels.best_per_row(x.shape[0], self.weight, x.dtype):
            return None
        return kernels.linear_best(x, self.weight)
