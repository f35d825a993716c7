"""Token embedding and LM head (reference: tinyvllm/layers/embed_head.py:9-70), one GPU."""
import torch
from torch import nn

from .. import ops
from ..utils.context import get_context
from .linear import StackedLinear


class VocabParallelEmbedding(nn.Module):
    def __init__(self, num_embeddings: int, embedding_dim: int):
        super().__init__()
        self.tp_rank, self.tp_size = 0, 1
        self.num_embeddings = num_embeddings
        self.num_embeddings_per_partition = num_embeddings
        self.weight = nn.Parameter(torch.empty(num_embeddings, embedding_dim))
        self.weight.weight_loader = self.weight_loader

    def weight_loader(self, param: nn.Parameter, loaded_weight: torch.Tensor):
        assert param.data.size() == loaded_weight.size()
        param.data.copy_(loaded_weight)

    def forward(self, x: torch.Tensor):
        return ops.embedding(x, self.weight.data)


class ParallelLMHead(VocabParallelEmbedding):
    def __init__(self, num_embeddings: int, embedding_dim: int, bias: bool = False):
        super().__init__(num_embeddings, embedding_dim)
        assert not bias

    @staticmethod
    def _wanted_rows(x: torch.Tensor):
        ctx = get_context()
        if ctx.logit_rows is not None:                       # the step says which rows
            return x[ctx.logit_rows].contiguous()
        if ctx.is_prefill:                                   # only the last token of each sequence
            last = (ctx.cu_seqlens_q[1:] - 1).long()
            x = x[last].contiguous()
        return x

    def forward(self, x: torch.Tensor):
        return ops.bf16_linear(self._wanted_rows(x), self.weight.data)

    def forward_greedy(self, x: torch.Tensor):
        """``argmax(self(x), -1)``: the greedy branch of the sampler (sampler.py:13-14,21) applied to this
        layer's logits, in one call that never stores them."""
        return ops.bf16_linear_argmax(self._wanted_rows(x), self.weight.data)


class PaddedLMHead(StackedLinear):
    """LM head of any vocabulary and width, bf16 or 32-bit."""

    def __init__(self, num_embeddings: int, embedding_dim: int):
        super().__init__(embedding_dim, {"head": num_embeddings})
        self.num_embeddings = num_embeddings

    def forward(self, x: torch.Tensor):
        return super().forward(ParallelLMHead._wanted_rows(x))[:, :self.num_embeddings]

    def forward_greedy(self, x: torch.Tensor):
        x = ParallelLMHead._wanted_rows(x)
        if self.weight.dtype == torch.bfloat16 and self.weight.shape == (self.num_embeddings, x.shape[-1]):
            return ops.bf16_linear_argmax(x, self.weight.data)
        return ops.argmax(super().forward(x)[:, :self.num_embeddings].contiguous())


class TiedLMHead(PaddedLMHead):
    """LM head on the embedding table: shares its memory where the sizes need no padding."""

    def tie_(self, table: torch.Tensor):
        if table.shape == self.weight.shape:
            self.weight.data = table
        else:
            self.weight.data[:table.shape[0], :table.shape[1]].copy_(table)
