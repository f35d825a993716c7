"""Softmax attention over latents, windowed or causal, on a paged cache of one row per token for all heads.

A token caches its normed latent and a rotated key part.  Decoded tokens, short portions and 32-bit mode attend in the
latent space: the queries are taken there once (``absorb``) and the mixed latents back to values once (``values``).  Long
portions expand the keys and values of every head with one product (``expand``) and attend on those."""
import torch
from torch import nn

from .. import ops
from ..utils.context import get_context


class LatentAttention(nn.Module):
    def __init__(self, num_heads: int, dim: int, rot_dim: int, rank: int, value_dim: int, scale: float, window: int,
                 window_index: int, rope, eps: float, dtype: torch.dtype, halves: bool = False):
        super().__init__()
        self.shape = ops.LatentShape(num_heads, dim, rot_dim, rank, value_dim)
        self.scale, self.window, self.window_index, self.eps, self.dtype = scale, window, window_index, eps, dtype
        self.halves = halves            # rotation of pairs (i, i + rot_dim / 2) instead of neighbours
        self.register_buffer("cos_sin", rope, persistent=False)
        self.norm = nn.Module()
        self.norm.weight = nn.Parameter(torch.ones(rank))
        self.uk = nn.Parameter(torch.zeros(num_heads * dim, rank))
        self.uv = nn.Parameter(torch.zeros(num_heads * value_dim, rank))
        self.absorb = self.values = self.expand = None      # made from uk and uv by pack_
        self.cache = None                                   # [pages, block, Lp], bound by the model runner

    # -- what the model runner asks a layer with a paged cache
    def page_bytes(self, block_size: int) -> int:
        return block_size * self.shape.lp * torch.empty(0, dtype=self.dtype).element_size()

    def bind_pages(self, pages: int, block_size: int, device):
        self.cache = torch.zeros(pages, block_size, self.shape.lp, dtype=self.dtype, device=device) if pages else None

    def pack_(self):
        """Once after loading: the three forms of the latent's projections."""
        s, new = self.shape, self.uk.new_zeros
        uk, uv = self.uk.data.view(s.heads, s.dim, s.rank), self.uv.data.view(s.heads, s.vdim, s.rank)
        # [q_own | q_rot] -> [Uk^T q_own | q_rot]: the rotated part passes through an identity
        self.absorb = new(s.heads, s.lp, s.dq)
        self.absorb[:, :s.rank, :s.dim] = uk.transpose(1, 2)
        for i in range(s.rot):
            self.absorb[:, s.ra + i, s.da + i] = 1
        self.values = new(s.heads, -(-s.vdim // 16) * 16, s.rp)
        self.values[:, :s.vdim, :s.rank] = uv
        self.tiles = self.dtype == torch.bfloat16 and ops.latent_attn_supported(s)
        if self.dtype == torch.bfloat16 and ops.latent_prefill_supported(s):
            rows = s.heads * (s.da + s.va)
            self.expand = new(-(-rows // 16) * 16, -(-s.ra // 64) * 64)
            self.expand[:s.heads * s.da].view(s.heads, s.da, -1)[:, :s.dim, :s.rank] = uk
            self.expand[s.heads * s.da:rows].view(s.heads, s.va, -1)[:, :s.vdim, :s.rank] = uv

    def prepare(self, proj, latent_col: int, positions: torch.Tensor) -> torch.Tensor:
        """Projection rows ``[q | ... | latent | rotated key]`` -> rotated queries; the new cache rows are stored."""
        return ops.latent_prep(proj, latent_col, self.norm.weight.data, positions, self.cos_sin, get_context().slot_mapping,
                               self.cache, self.shape, self.eps)

    def prepare_down(self, proj, latent_col: int, positions: torch.Tensor, cq_col: int, cq_norm, gate_col: int):
        """Rows ``[query latent | latent | rotated key | gate]`` at their columns -> normed query latents, gates; the new cache rows
        are stored."""
        return ops.latent_prep_down(proj, latent_col, self.norm.weight.data, positions, self.cos_sin, get_context().slot_mapping, self.cache,
                                    self.shape, self.eps, self.halves, cq_col, cq_norm, gate_col)

    def prepare_queries(self, proj, positions: torch.Tensor) -> torch.Tensor:
        return ops.latent_prep_queries(proj, positions, self.cos_sin, self.shape, self.halves)

    def forward(self, q, positions: torch.Tensor, out: torch.Tensor, gate=None):
        """Queries from ``prepare`` -> ``out[:, :heads * value_dim]``, a head's result times its ``gate`` (fp32 ``[N, heads]``)."""
        ctx, n = get_context(), q.shape[0]
        latent_rows = ctx.num_short_rows if self.expand is not None else n
        if latent_rows:
            self._latent(q[:latent_rows], positions[:latent_rows], out[:latent_rows], gate[:latent_rows] if gate is not None else None)
        if latent_rows < n:
            self._expanded(q, out, gate)

    def _latent(self, q, positions, out, gate):
        ctx, s, n = get_context(), self.shape, q.shape[0]
        q = ops.head_gemm(q, self.absorb, s.ra, -(-s.da // 32) * 32)
        if not self.tiles:
            part, ml = ops.latent_rows(q, self.cache, ctx.block_tables, positions, ctx.slot_mapping[:n],
                                       ctx.row_seq[:n] if ctx.row_seq is not None else None, self.window, self.scale, s)
            ops.latent_values(part, ml, self.values, out, s, gate=gate)
            return
        single, short = ctx.num_single, self.expand is not None
        if single:
            batch = ops.LatentBatch(single, positions=positions, slot_mapping=ctx.slot_mapping)
            self._tiles(q[:single], "single", batch, out[:single], gate[:single] if gate is not None else None)
        if single < n:
            batch = ops.LatentBatch(ctx.num_short if short else ctx.cu_seqlens_q.numel() - 1 - single,
                                    ctx.max_short if short else ctx.max_portion, cu_seqlens_q=ctx.cu_seqlens_q,
                                    seq_starts=ctx.seq_starts, row_seq=ctx.row_seq[single:n], first_seq=single, first_row=single)
            self._tiles(q[single:], "portions", batch, out[single:], gate[single:] if gate is not None else None)

    def _tiles(self, q, kind: str, batch, out, gate):
        ctx, s = get_context(), self.shape
        key = (kind, s.heads, s.lp, self.window)           # layers of these sizes share a step's plan
        if key not in ctx.plans:
            ctx.plans[key] = ops.latent_plan(batch, s.heads, s.lp, self.window)
        plan = ctx.plans[key]
        part, ml = ops.latent_attention(q, self.cache, ctx.block_tables, self.window, self.scale, s, batch, plan)
        ops.latent_values(part, ml, self.values, out, s, batch, plan, gate)

    def _expanded(self, q, out, gate):
        ctx, w = get_context(), self.window_index
        first = ctx.num_single + ctx.num_short
        seqs = ctx.cu_seqlens_q.numel() - 1 - first
        offsets = ctx.kv_offsets[w]
        latents = ops.latent_gather(self.cache, ctx.block_tables, ctx.cu_seqlens_q, ctx.seq_starts, offsets, ctx.kv_rows[w],
                                    first, seqs, ctx.max_kv_rows[w], self.window)
        expanded = ops.linear(latents[:, :self.expand.shape[1]], self.expand)
        ops.latent_prefill(q, expanded, latents, ctx.cu_seqlens_q, ctx.seq_starts, offsets, first, seqs, ctx.max_portion,
                           self.window, self.scale, self.shape, out, gate)
