"""Vocab-parallel embedding and LM head.

Parity: layers/vocab_parallel_embedding.py (vocab padded to 64, shard
mask + all-reduce for the embedding; logits all-gather for the head).
"""

import torch
import torch.nn as nn
import torch.nn.functional as F

from gllm_amd.parallel import (get_tp_rank, get_tp_size,
                               tensor_parallel_all_gather,
                               tensor_parallel_all_reduce)


def pad_vocab(vocab_size: int, align: int = 64) -> int:
    return -(-vocab_size // align) * align


class VocabParallelEmbedding(nn.Module):
    def __init__(self, vocab_size: int, hidden_size: int, params_dtype=None):
        super().__init__()
        tp = get_tp_size()
        self.vocab_size = vocab_size
        self.padded_vocab = pad_vocab(vocab_size, 64 * tp)
        self.shard_size = self.padded_vocab // tp
        self.vocab_start = get_tp_rank() * self.shard_size
        self.vocab_end = self.vocab_start + self.shard_size
        dtype = params_dtype or torch.get_default_dtype()
        self.weight = nn.Parameter(
            torch.empty(self.shard_size, hidden_size, dtype=dtype),
            requires_grad=False)
        self.weight.weight_loader = self._load

    def _load(self, param, loaded):
        n = min(self.shard_size, max(0, loaded.shape[0] - self.vocab_start))
        param.data.zero_()
        if n > 0:
            param.data[:n].copy_(loaded.narrow(0, self.vocab_start, n))

    def forward(self, input_ids: torch.Tensor) -> torch.Tensor:
        if get_tp_size() == 1:
            return F.embedding(input_ids, self.weight)
        mask = (input_ids >= self.vocab_start) & (input_ids < self.vocab_end)
        local = (input_ids - self.vocab_start).clamp_(0, self.shard_size - 1)
        emb = F.embedding(local, self.weight)
        emb = emb * mask.unsqueeze(-1).to(emb.dtype)
        return tensor_parallel_all_reduce(emb)


class NormedEmbedding(VocabParallelEmbedding):
    """Token embedding that opens an fp32 residual stream:

        x = RMSnorm(weight[id] * scale + positions[p]) * norm

    with an optional learned position table (``max_positions`` rows; 0 =
    none) and a norm weight stored as its distance from
    ``weight_offset``. ``forward`` returns (x in fp32, x in the model
    dtype); one launch on the GPU (ops.embed_rmsnorm). One rank only:
    the norm needs the whole row."""

    def __init__(self, vocab_size: int, hidden_size: int, eps: float,
                 scale: float = 1.0, max_positions: int = 0,
                 weight_offset: float = 0.0, params_dtype=None):
        super().__init__(vocab_size, hidden_size, params_dtype)
        assert get_tp_size() == 1
        dtype = self.weight.dtype
        self.scale, self.eps = float(scale), eps
        self.weight_offset = float(weight_offset)
        self.norm_weight = nn.Parameter(
            torch.full((hidden_size,), 1.0 - self.weight_offset,
                       dtype=dtype), requires_grad=False)
        if max_positions:
            self.positions = nn.Parameter(
                torch.zeros(max_positions, hidden_size, dtype=dtype),
                requires_grad=False)
        else:
            self.register_parameter("positions", None)

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor):
        from gllm_amd import ops
        return ops.embed_rmsnorm(input_ids, positions, self.weight,
                                 self.positions, self.norm_weight,
                                 self.scale, self.weight_offset, self.eps)


class TokenSideInput(nn.Module):
    """A per-token, per-layer input of low width:

        y = proj(gelu_tanh(gate(h)) * table[id, col0:col0 + dim])

    ``table`` [vocab, layers * dim] is shared by the layers and passed
    per call; the caller owns the norm of y and its place in the
    stream."""

    def __init__(self, hidden_size: int, dim: int, layer_idx: int,
                 params_dtype=None):
        super().__init__()
        from gllm_amd.layers.linear import ReplicatedLinear
        self.col0 = layer_idx * dim
        self.gate = ReplicatedLinear(hidden_size, dim,
                                     params_dtype=params_dtype)
        self.proj = ReplicatedLinear(dim, hidden_size,
                                     params_dtype=params_dtype)

    def forward(self, h: torch.Tensor, input_ids: torch.Tensor,
                table: torch.Tensor) -> torch.Tensor:
        from gllm_amd import ops
        return self.proj(ops.token_gate(self.gate(h), table, input_ids,
                                        self.col0))


class ParallelLMHead(nn.Module):
    """Logits = H @ W_shard^T, all-gathered to the full padded vocab."""

    def __init__(self, vocab_size: int, hidden_size: int, bias: bool = False,
                 params_dtype=None):
        super().__init__()
        tp = get_tp_size()
        self.vocab_size = vocab_size
        self.padded_vocab = pad_vocab(vocab_size, 64 * tp)
        self.shard_size = self.padded_vocab // tp
        self.vocab_start = get_tp_rank() * self.shard_size
        dtype = params_dtype or torch.get_default_dtype()
        self.weight = nn.Parameter(
            torch.empty(self.shard_size, hidden_size, dtype=dtype),
            requires_grad=False)
        self.weight.weight_loader = self._load

    def _load(self, param, loaded):
        n = min(self.shard_size, max(0, loaded.shape[0] - self.vocab_start))
        param.data.zero_()
        if n > 0:
            param.data[:n].copy_(loaded.narrow(0, self.vocab_start, n))

    def tie_to(self, embedding: VocabParallelEmbedding):
        self.weight = embedding.weight

    def forward(self, hidden: torch.Tensor) -> torch.Tensor:
        from gllm_amd import ops
        logits = ops.linear(hidden, self.weight)
        if get_tp_size() > 1:
            logits = tensor_parallel_all_gather(logits, dim=-1)
        return logits[..., :self.vocab_size]
