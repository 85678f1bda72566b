"""Minimal continuous-batching attention engine over the paged KV cache.

What a KV-cached replacement of TransformerLM.generate (llm-core/llm_core/model.py:187-236,
which re-runs the whole forward per token at :218) needs around the attention kernels: a block
allocator, per-sequence block tables, slot mapping for cache writes, a prefill call for newly
admitted sequences and a decode call that serves every running sequence with one kernel launch
per layer and step.  The bookkeeping (blocks, lengths, tables) is shared by all attention layers
of a model; every layer has its own K/V pools, of its own head count and head sizes, or reads those
of an earlier layer (`AttentionLayer`); a recurrent layer has a fixed-size state per sequence instead, in the sequence's
state slot (`StateLayer`).  A step is planned once (`plan_prefill`,
`plan_decode`: host integers -> a few small device tensors) and then applied per layer
(`attend_prefill`, `attend_decode`, `advance_state`).  Projections, sampling and the scheduler policy stay with
the caller.

All tensor work runs on the HIP kernels (rope_and_cache, rope_rotate, kv_cache_write, flash_attn_varlen_prefill,
flash_attn_paged_prefill, paged_attention_decode, paged_attention_any, ssm_mix); the bookkeeping here is plain Python on host integers.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, field

import torch

from . import ops

BLOCK = 16


class OutOfBlocks(RuntimeError):
    pass


@dataclass
class AttentionLayer:
    """One attention layer as the cache manager sees it.  head_dim is the size of a query/key head, v_dim of a value
    head (None: head_dim).  kv_from = i: the layer has no keys and values of its own and reads layer i's pools.
    softmax_scale None: 1/sqrt(head_dim).  head_scale (non-negative factor per query head) and sinks (score without key
    or value per query head) are fp32 (n_q_heads,) tensors or None.  rope: rotate adjacent pairs of q and k by the position;
    rope_base None: with the engine's rope_theta over the whole head, else the first rope_dims (None: all) entries of a head
    turn, pair i by rope_base^(-2i/rope_dims) per position.  window > 0: the token at position i sees position j when i - j <
    window or j < keep_first."""
    n_q_heads: int
    n_kv_heads: int
    head_dim: int
    v_dim: int | None = None
    kv_from: int | None = None
    softmax_scale: float | None = None
    head_scale: torch.Tensor | None = None
    sinks: torch.Tensor | None = None
    rope: bool = True
    rope_base: float | None = None
    rope_dims: int | None = None
    window: int = 0
    keep_first: int = 0


@dataclass
class StateLayer:
    """One Mamba-2 mixer as the state manager sees it: per sequence the last `taps` inputs of its convolution and, in fp32, a
    (state x vdim) matrix per head.  params: the fp32 tensors that ops.ssm_mix takes."""
    heads: int
    vdim: int
    state: int
    groups: int
    taps: int
    params: dict

    @property
    def channels(self) -> int:
        return self.heads * self.vdim + 2 * self.groups * self.state


def cache_head_dims(kv_dtype: str, head_dim: int, v_dim: int) -> tuple[int, int, bool]:
    """(key size, value size, mfma?) of the head rows a pool holds.  The MFMA kernels take equal sizes of 32, 64 or 128
    (fp8: 64 or 128): smaller heads are padded with zeros up to the next of these, which changes neither a score nor a
    sum.  fp32 pools and larger heads go to the general kernel, in rows of whole 8-element pieces."""
    if kv_dtype != "fp32":
        for d in ((64, 128) if kv_dtype == "fp8" else (32, 64, 128)):
            if max(head_dim, v_dim) <= d:
                return d, d, True
    if kv_dtype == "fp8":
        raise ValueError("an fp8 KV cache needs head sizes up to 128")
    if max(head_dim, v_dim) > 512:
        raise ValueError("head sizes above 512 are not supported")
    return (head_dim + 7) // 8 * 8, (v_dim + 7) // 8 * 8, False


class BlockAllocator:
    """Free list of physical cache blocks."""

    def __init__(self, num_blocks: int):
        self.num_blocks = num_blocks
        self._free = list(range(num_blocks - 1, -1, -1))

    @property
    def num_free(self) -> int:
        return len(self._free)

    def allocate(self) -> int:
        if not self._free:
            raise OutOfBlocks("KV cache is out of blocks")
        return self._free.pop()

    def free(self, blocks) -> None:
        self._free.extend(blocks)


@dataclass
class PrefillPlan:
    positions: torch.Tensor      # (T,) int32
    slots: torch.Tensor          # (T,) int64
    cu_seqlens: torch.Tensor     # (B+1,) int32
    max_len: int
    last_rows: torch.Tensor      # (B,) int64: packed row of each sequence's last token
    # set when some sequence already had tokens in the cache (a further chunk of its prompt): the attention
    # then reads all keys and values through the block tables
    tables: torch.Tensor | None = None        # (B, max_blocks) int32
    context_lens: torch.Tensor | None = None  # (B,) int32: tokens in the cache, this chunk included
    total_context: int = 0                    # their sum (sizes the dequantised rows of an fp8 cache)
    cu_context: torch.Tensor | None = None    # (B+1,) int32: their running sum (fp8 cache: where each sequence's rows start)
    state_slots: torch.Tensor | None = None   # (B,) int32: where each sequence's recurrent state lives
    # packed keys and values of layers that later layers share (new sequences only), by layer
    packed: dict[int, tuple] = field(default_factory=dict)


@dataclass
class DecodePlan:
    positions: torch.Tensor      # (B,) int32
    slots: torch.Tensor          # (B,) int64
    tables: torch.Tensor         # (B, max_blocks) int32
    context_lens: torch.Tensor   # (B,) int32, the new token included
    max_context: int
    state_slots: torch.Tensor | None = None      # (B,) int32


class StaticDecodeStep:
    """Device tensors of one decode step at fixed addresses, refreshed from the host by one copy.

    Layout of the int32 buffer: token ids (int64), slots (int64), positions, context lengths,
    state slots, block tables (batch x max_blocks)."""

    def __init__(self, batch: int, max_blocks: int, device):
        B, M = batch, max_blocks
        self.batch, self.max_blocks = B, M
        n = 7 * B + B * M
        self._dev = torch.zeros(n, dtype=torch.int32, device=device)
        self._host = torch.zeros(n, dtype=torch.int32, pin_memory=True)
        self._copied = torch.cuda.Event()
        self._pending = False
        self.tokens = self._dev[0:2 * B].view(torch.int64)
        slots = self._dev[2 * B:4 * B].view(torch.int64)
        positions = self._dev[4 * B:5 * B]
        context_lens = self._dev[5 * B:6 * B]
        tables = self._dev[7 * B:].view(B, M)
        self.plan = DecodePlan(positions, slots, tables, context_lens, M * BLOCK, self._dev[6 * B:7 * B])
        h = self._host
        self._h_tokens, self._h_slots = h[0:2 * B].view(torch.int64), h[2 * B:4 * B].view(torch.int64)
        self._h_positions, self._h_ctx, self._h_state = h[4 * B:5 * B], h[5 * B:6 * B], h[6 * B:7 * B]
        self._h_tables = h[7 * B:].view(B, M)

    def fill(self, tokens, slots, positions, context_lens, block_lists, state_slots) -> None:
        if self._pending:
            self._copied.synchronize()              # the previous copy has left the staging buffer
        self._h_tokens.copy_(torch.tensor(tokens, dtype=torch.int64))
        self._h_slots.copy_(torch.tensor(slots, dtype=torch.int64))
        self._h_positions.copy_(torch.tensor(positions, dtype=torch.int32))
        self._h_ctx.copy_(torch.tensor(context_lens, dtype=torch.int32))
        self._h_state.copy_(torch.tensor(state_slots, dtype=torch.int32))
        for i, blocks in enumerate(block_lists):
            self._h_tables[i, :len(blocks)] = torch.tensor(blocks, dtype=torch.int32)
        self._dev.copy_(self._host, non_blocking=True)
        self._copied.record()
        self._pending = True


class PagedAttentionEngine:
    def __init__(self, num_blocks, n_q_heads=None, n_kv_heads=None, head_dim=None, context_length=None, *, rope_theta=10000.0,
                 max_batch=256, num_layers=1, kv_dtype="bf16", device="cuda:0",
                 layers: list[AttentionLayer | StateLayer] | None = None):
        """Either n_q_heads, n_kv_heads, head_dim and num_layers (equal layers with RoPE) or `layers`.  kv_dtype: "bf16",
        "fp8" (e4m3 + scales) or "fp32" (pools, queries and outputs in fp32, general attention kernel).
        q, k and v of layer i come with the head sizes cache_dims[i] (padded with zeros where a head is smaller).  With state
        layers at most max_batch sequences exist at a time."""
        self.device = torch.device(device)
        if context_length is None:
            raise ValueError("context_length is required")
        if kv_dtype not in ("bf16", "fp8", "fp32"):
            raise ValueError("kv_dtype must be 'bf16', 'fp8' or 'fp32'")
        if layers is None:
            if kv_dtype == "fp8" and head_dim not in (64, 128):
                raise ValueError("an fp8 KV cache needs head_dim 64 or 128")
            if kv_dtype == "fp32":
                raise ValueError("an fp32 KV cache has no rotating cache write; describe layers without rope")
            layers = [AttentionLayer(n_q_heads, n_kv_heads, head_dim) for _ in range(num_layers)]
        self.layers = layers
        self.num_layers = len(layers)
        self.context_length = context_length
        self.kv_dtype = kv_dtype
        attention = [ly for ly in layers if isinstance(ly, AttentionLayer)]
        if attention:
            self.Hq, self.Hkv, self.D = attention[0].n_q_heads, attention[0].n_kv_heads, attention[0].head_dim
        cache_dtype = {"bf16": torch.bfloat16, "fp8": torch.uint8, "fp32": torch.float32}[kv_dtype]      # uint8 = e4m3 bit patterns
        self.k_caches, self.v_caches, self.cache_dims, self.mfma = [], [], [], []
        # per-(block, kv head) scales of an fp8 cache, maintained by the cache write
        self.k_scales, self.v_scales = ([], []) if kv_dtype == "fp8" else (None, None)
        self.shared = {ly.kv_from for ly in attention if ly.kv_from is not None}
        self.conv_states, self.ssm_states = {}, {}        # by state layer
        rope_dims, tables = set(), {}
        self.freq_caches = []                             # by layer: its cos/sin table or None
        for i, ly in enumerate(layers):
            if isinstance(ly, StateLayer):
                act = torch.float32 if kv_dtype == "fp32" else torch.bfloat16
                self.conv_states[i] = torch.zeros(max_batch, ly.taps, ly.channels, dtype=act, device=self.device)
                self.ssm_states[i] = torch.zeros(max_batch, ly.heads, ly.state, (ly.vdim + 3) // 4 * 4, dtype=torch.float32,
                                                 device=self.device)
                for per_layer in (self.k_caches, self.v_caches, self.cache_dims, self.mfma, self.freq_caches):
                    per_layer.append(None)
                if kv_dtype == "fp8":
                    self.k_scales.append(None)
                    self.v_scales.append(None)
                continue
            if ly.n_q_heads < 1 or ly.n_kv_heads < 1 or ly.n_q_heads % ly.n_kv_heads:
                raise ValueError(f"layer {i}: {ly.n_q_heads} query heads over {ly.n_kv_heads} kv heads")
            kd, vd, mfma = cache_head_dims(kv_dtype, ly.head_dim, ly.v_dim or ly.head_dim)
            if ly.rope and ly.rope_base is None and (not mfma or kd != ly.head_dim or (ly.v_dim or kd) != kd):
                raise ValueError(f"layer {i}: RoPE needs equal head sizes of 32, 64 or 128 and a 16- or 8-bit cache")
            if ly.window < 0 or ly.keep_first < 0:
                raise ValueError(f"layer {i}: window and keep_first must not be negative")
            self.cache_dims.append((kd, vd))
            self.mfma.append(mfma)
            src = ly.kv_from
            if src is not None:
                if not 0 <= src < i or not isinstance(layers[src], AttentionLayer) or layers[src].kv_from is not None:
                    raise ValueError(f"layer {i}: kv_from {src} is not an earlier layer with keys and values of its own")
                if layers[src].n_kv_heads != ly.n_kv_heads or self.cache_dims[src] != (kd, vd) \
                        or any(getattr(layers[src], n) != getattr(ly, n) for n in ("rope", "rope_base", "rope_dims")):
                    raise ValueError(f"layer {i}: kv heads, head sizes and rotation differ from those of layer {src}, whose cache it reads")
                self.k_caches.append(self.k_caches[src])
                self.v_caches.append(self.v_caches[src])
            else:
                self.k_caches.append(torch.zeros(num_blocks, ly.n_kv_heads, BLOCK, kd, dtype=cache_dtype, device=self.device))
                self.v_caches.append(torch.zeros(num_blocks, ly.n_kv_heads, BLOCK, vd, dtype=cache_dtype, device=self.device))
            if kv_dtype == "fp8":
                for sc in (self.k_scales, self.v_scales):
                    sc.append(sc[src] if src is not None else
                              torch.ones(num_blocks, ly.n_kv_heads, dtype=torch.float32, device=self.device))
            key = None
            if ly.rope and ly.rope_base is None:
                rope_dims.add(kd)
                key = kd
                if key not in tables:
                    tables[key] = ops.build_rope_cache(context_length, kd, rope_theta, self.device)
            elif ly.rope:
                key = (kd, ly.head_dim if ly.rope_dims is None else ly.rope_dims, float(ly.rope_base))
                if key not in tables:
                    tables[key] = ops.build_partial_rope_cache(context_length, *key, self.device)
            self.freq_caches.append(tables.get(key))
        # layers on the general kernel read every key through the tables, also in the first chunk of a prompt
        self.always_tables = any(m is False for m in self.mfma)
        if len(rope_dims) > 1:
            raise ValueError("layers with RoPE must share one head size")
        self.freq_cache = next((t for t in self.freq_caches if t is not None), None)
        # rotation by the angle 0 (cos 1, sin 0, every position clamped to the one row) for layers without RoPE on an fp8 cache
        self._no_rotation = {d: torch.stack((torch.ones(1, d // 2), torch.zeros(1, d // 2))).to(self.device)
                             for d in {dims[0] for dims in self.cache_dims if dims}} if kv_dtype == "fp8" else None
        self.allocator = BlockAllocator(num_blocks)
        self.blocks: dict[int, list[int]] = {}      # sequence id -> physical blocks
        self.lengths: dict[int, int] = {}           # sequence id -> tokens in the cache
        self.state_slots: dict[int, int] = {}       # sequence id -> state slot (models with state layers)
        self._free_slots = list(range(max_batch - 1, -1, -1))
        self.max_blocks_per_seq = (context_length + BLOCK - 1) // BLOCK
        # persistent step buffers: no allocation on the decode path besides the kernel outputs
        self._tables = torch.zeros(max_batch, self.max_blocks_per_seq, dtype=torch.int32, device=self.device)
        self._workspace = max((ops.paged_decode_workspace(max_batch, hq, d, context_length, self.device)
                               for hq, d in {(ly.n_q_heads, dims[0]) for ly, dims, m in zip(layers, self.cache_dims, self.mfma) if m}),
                              key=lambda t: t.numel(), default=None)
        self.max_batch = max_batch

    # the pools of layer 0 under their single-layer names
    @property
    def k_cache(self):
        return self.k_caches[0]

    @property
    def v_cache(self):
        return self.v_caches[0]

    # ---- bookkeeping ---------------------------------------------------------
    def add_sequence(self, seq_id: int) -> None:
        if seq_id in self.blocks:
            raise ValueError(f"sequence {seq_id} already exists")
        if self.conv_states:
            if not self._free_slots:
                raise OutOfBlocks(f"all {self.max_batch} state slots are taken")
            self.state_slots[seq_id] = self._free_slots.pop()
        self.blocks[seq_id] = []
        self.lengths[seq_id] = 0

    def remove_sequence(self, seq_id: int) -> None:
        self.allocator.free(self.blocks.pop(seq_id))
        del self.lengths[seq_id]
        if seq_id in self.state_slots:
            self._free_slots.append(self.state_slots.pop(seq_id))       # (a new sequence starts from zero whatever the slot holds)

    def _slots_of(self, seq_ids) -> torch.Tensor | None:
        return torch.tensor([self.state_slots[s] for s in seq_ids], dtype=torch.int32, device=self.device) if self.conv_states else None

    def _reserve(self, seq_id: int, n_new: int) -> list[int]:
        """Slots for the next n_new tokens of a sequence (allocates blocks as needed)."""
        length = self.lengths[seq_id]
        if length + n_new > self.context_length:
            raise ValueError(f"sequence {seq_id} would exceed context_length {self.context_length}")
        blocks = self.blocks[seq_id]
        need = (length + n_new + BLOCK - 1) // BLOCK - len(blocks)
        if need > self.allocator.num_free:
            raise OutOfBlocks(f"sequence {seq_id} needs {need} blocks, {self.allocator.num_free} free")
        for _ in range(need):
            blocks.append(self.allocator.allocate())
        slots = [blocks[t // BLOCK] * BLOCK + t % BLOCK for t in range(length, length + n_new)]
        self.lengths[seq_id] = length + n_new
        return slots

    # ---- planning (once per step) ---------------------------------------------
    def plan_prefill(self, seq_ids, lens) -> PrefillPlan:
        """Reserves cache slots for the next `lens[i]` prompt tokens of each sequence in `seq_ids`.  A sequence
        may be new (the usual case) or already hold tokens -- a further chunk of a long prompt, or a prompt on
        top of a cached prefix: the chunk's queries then attend to everything cached so far (with an fp8 cache: to
        the quantised keys and values, the chunk's own included, as every later decode step will)."""
        if len(seq_ids) != len(lens) or not seq_ids:
            raise ValueError("seq_ids and lens must be non-empty and of equal length")
        if len(set(seq_ids)) != len(seq_ids):
            raise ValueError("a sequence may appear only once per prefill")
        for sid, n in zip(seq_ids, lens):
            if n < 1 or self.lengths[sid] + n > self.context_length:
                raise ValueError(f"prompt lengths must be in 1..{self.context_length} (tokens already cached included)")
        chunked = any(self.lengths[sid] != 0 for sid in seq_ids)
        need = sum((self.lengths[sid] + n + BLOCK - 1) // BLOCK - len(self.blocks[sid]) for sid, n in zip(seq_ids, lens))
        if need > self.allocator.num_free:
            raise OutOfBlocks(f"prefill needs {need} blocks, {self.allocator.num_free} free")
        slots, positions, cu = [], [], [0]
        for sid, n in zip(seq_ids, lens):
            start = self.lengths[sid]
            slots += self._reserve(sid, n)
            positions += list(range(start, start + n))
            cu.append(cu[-1] + n)
        dev = self.device
        plan = PrefillPlan(torch.tensor(positions, dtype=torch.int32, device=dev),
                           torch.tensor(slots, dtype=torch.int64, device=dev),
                           torch.tensor(cu, dtype=torch.int32, device=dev), max(lens),
                           torch.tensor([c - 1 for c in cu[1:]], dtype=torch.int64, device=dev),
                           state_slots=self._slots_of(seq_ids))
        if chunked or self.always_tables:
            max_blk = max(len(self.blocks[sid]) for sid in seq_ids)
            rows = torch.zeros(len(seq_ids), max_blk, dtype=torch.int32)
            for i, sid in enumerate(seq_ids):
                b = self.blocks[sid]
                rows[i, :len(b)] = torch.tensor(b, dtype=torch.int32)
            plan.tables = rows.to(dev)
            plan.context_lens = torch.tensor([self.lengths[sid] for sid in seq_ids], dtype=torch.int32, device=dev)
            plan.total_context = sum(self.lengths[sid] for sid in seq_ids)
            if self.kv_dtype == "fp8":
                run = [0]
                for sid in seq_ids:
                    run.append(run[-1] + self.lengths[sid])
                plan.cu_context = torch.tensor(run, dtype=torch.int32, device=dev)
        return plan

    def _reserve_decode(self, seq_ids):
        """Host side of a decode step: checks, reserves one slot per sequence.  Returns (positions, slots)."""
        B = len(seq_ids)
        if B == 0 or B > self.max_batch:
            raise ValueError(f"batch {B} must be in 1..{self.max_batch}")
        if len(set(seq_ids)) != B:
            raise ValueError("a sequence may appear only once per decode step")
        for s in seq_ids:
            if self.lengths[s] == 0:
                raise ValueError(f"sequence {s} has no tokens; prefill it first")
            if self.lengths[s] + 1 > self.context_length:
                raise ValueError(f"sequence {s} would exceed context_length {self.context_length}")
        need = sum(1 for s in seq_ids if self.lengths[s] % BLOCK == 0)
        if need > self.allocator.num_free:
            raise OutOfBlocks(f"decode step needs {need} blocks, {self.allocator.num_free} free")
        positions = [self.lengths[s] for s in seq_ids]
        slots = [self._reserve(s, 1)[0] for s in seq_ids]
        return positions, slots

    def plan_decode(self, seq_ids) -> DecodePlan:
        """Reserves the slot of one new token for each running sequence in `seq_ids`."""
        B = len(seq_ids)
        positions, slots = self._reserve_decode(seq_ids)
        dev = self.device
        max_len = max(self.lengths[s] for s in seq_ids)
        max_blk = (max_len + BLOCK - 1) // BLOCK
        rows = torch.zeros(B, max_blk, dtype=torch.int32)
        for i, s in enumerate(seq_ids):
            b = self.blocks[s]
            rows[i, :len(b)] = torch.tensor(b, dtype=torch.int32)
        tables = self._tables[:B, :max_blk]
        tables.copy_(rows, non_blocking=False)
        return DecodePlan(torch.tensor(positions, dtype=torch.int32, device=dev),
                          torch.tensor(slots, dtype=torch.int64, device=dev), tables,
                          torch.tensor([p + 1 for p in positions], dtype=torch.int32, device=dev), max_blk * BLOCK,
                          self._slots_of(seq_ids))

    def make_static_decode(self, batch: int) -> "StaticDecodeStep":
        """Fixed device tensors for decode steps of `batch` sequences (what a captured HIP graph needs:
        the same addresses and shapes on every replay)."""
        if batch < 1 or batch > self.max_batch:
            raise ValueError(f"batch {batch} must be in 1..{self.max_batch}")
        return StaticDecodeStep(batch, self.max_blocks_per_seq, self.device)

    def plan_decode_into(self, seq_ids, tokens, static: "StaticDecodeStep") -> DecodePlan:
        """plan_decode whose tensors (and the new token ids) are written into `static`: one pinned staging
        buffer, one asynchronous copy on the current stream.  Tables have their full width and
        max_context is the context length, so nothing about the step's shapes depends on the data."""
        B = len(seq_ids)
        if B != static.batch or len(tokens) != B:
            raise ValueError("seq_ids, tokens and the static buffers disagree on the batch size")
        positions, slots = self._reserve_decode(seq_ids)
        static.fill([int(t) for t in tokens], slots, positions, [p + 1 for p in positions],
                    [self.blocks[s] for s in seq_ids], [self.state_slots.get(s, 0) for s in seq_ids])
        return static.plan

    # ---- attention calls (once per layer) -----------------------------------------
    def _write_cache(self, layer: int, plan, q, k, v, k_out=None):
        """q and k rotated (layers with RoPE), k and v into layer `layer`'s cache (quantised when the cache is fp8);
        returns the query to attend with -- with k_out=True the pair (query, keys in packed form).  A layer that reads
        another layer's cache (k and v None) writes nothing."""
        if self.layers[layer].kv_from is not None:
            if k is not None or v is not None:
                raise ValueError(f"layer {layer} reads the cache of layer {self.layers[layer].kv_from} and takes no keys or values")
            return (q, None) if k_out else q
        kc, vc = self.k_caches[layer], self.v_caches[layer]
        rope = self.layers[layer].rope
        if rope and (not self.mfma[layer] or self.cache_dims[layer][0] != self.cache_dims[layer][1]):
            ops.rope_rotate(q, k, plan.positions, self.freq_caches[layer])          # (in place)
            rope = False
        if self.kv_dtype == "fp8":
            freq = self.freq_caches[layer] if rope else self._no_rotation[q.shape[2]]
            return ops.rope_and_cache_fp8(q, k, v, plan.positions, freq, kc, vc, self.k_scales[layer],
                                          self.v_scales[layer], plan.slots, k_out=k_out)
        if rope:
            return ops.rope_and_cache(q, k, v, plan.positions, self.freq_caches[layer], kc, vc, plan.slots, k_out=k_out)
        ops.kv_cache_write(k, v, kc, vc, plan.slots)
        return (q, k) if k_out else q

    def _score_terms(self, layer: int):
        ly = self.layers[layer]
        scale = 1.0 / math.sqrt(ly.head_dim) if ly.softmax_scale is None else ly.softmax_scale        # (of the unpadded head)
        return dict(softmax_scale=scale, head_scale=ly.head_scale, sinks=ly.sinks, window=ly.window, keep_first=ly.keep_first)

    def attend_prefill(self, layer: int, plan: PrefillPlan, q, k, v, out=None):
        """q (T,Hq,D), k/v (T,Hkv,D) packed along dim 0 (token strides free, heads contiguous; k and v None for a layer
        that reads another layer's cache).  Writes (rotated) K and V of layer `layer` into its cache and returns causal
        attention output (T,Hq,D).  New sequences attend to the packed tensors themselves; when a sequence already had
        cached tokens, keys and values are read back through the block tables, old and new alike.  out: where to write (rows may
        be strided)."""
        if q.shape[0] != plan.positions.shape[0]:
            raise ValueError("the plan and the packed tensors disagree on the number of tokens")
        terms = dict(self._score_terms(layer), out=out)
        if plan.tables is not None:
            q = self._write_cache(layer, plan, q, k, v)
            kc, vc = self.k_caches[layer], self.v_caches[layer]
            if not self.mfma[layer]:
                return ops.paged_attention_any(q, kc, vc, plan.tables, plan.context_lens, cu_seqlens_q=plan.cu_seqlens, **terms)
            if self.kv_dtype == "fp8":
                terms.update(k_scale=self.k_scales[layer], v_scale=self.v_scales[layer], total_context=plan.total_context,
                             cu_seqlens_k=plan.cu_context)
            return ops.flash_attn_paged_prefill(q, kc, vc, plan.cu_seqlens, plan.tables, plan.context_lens, plan.max_len, **terms)
        q, k = self._write_cache(layer, plan, q, k, v, k_out=True)
        src = self.layers[layer].kv_from
        if src is not None:
            k, v = plan.packed[src]
        elif layer in self.shared:
            plan.packed[layer] = (k, v)
        return ops.flash_attn_varlen_prefill(q, k, v, plan.cu_seqlens, plan.cu_seqlens, plan.max_len,
                                             plan.max_len, causal=True, **terms)

    def attend_decode(self, layer: int, plan: DecodePlan, q, k, v, out=None):
        """q (B,Hq,D), k/v (B,Hkv,D) or None as in attend_prefill: appends the token's K/V to layer `layer`'s cache and
        returns its attention output (B,Hq,D), written into `out` when given (rows may be strided)."""
        if q.shape[0] != plan.positions.shape[0]:
            raise ValueError("one query token per sequence expected")
        q = self._write_cache(layer, plan, q, k, v)
        terms = dict(self._score_terms(layer), out=out)
        kc, vc = self.k_caches[layer], self.v_caches[layer]
        if not self.mfma[layer]:
            return ops.paged_attention_any(q, kc, vc, plan.tables, plan.context_lens, **terms)
        if self.kv_dtype == "fp8":
            terms.update(k_scale=self.k_scales[layer], v_scale=self.v_scales[layer])
        return ops.paged_attention_decode(q, kc, vc, plan.tables, plan.context_lens, max_context=plan.max_context,
                                          workspace=self._workspace, **terms)

    def advance_state(self, layer: int, plan: PrefillPlan | DecodePlan, proj, xbc_col: int, dt_col: int, out=None):
        """State layer `layer` over the plan's tokens: the columns of proj (T,*) that hold its convolution inputs and step sizes
        (see ops.ssm_mix), each sequence's state read from its slot and left there.  Returns y (T, heads * vdim)."""
        ly = self.layers[layer]
        if proj.shape[0] != plan.positions.shape[0]:
            raise ValueError("the plan and the projection disagree on the number of tokens")
        return ops.ssm_mix(proj, xbc_col, dt_col, ly.params, self.conv_states[layer], self.ssm_states[layer], plan.state_slots,
                           plan.positions, plan.cu_seqlens if isinstance(plan, PrefillPlan) else None, heads=ly.heads, vdim=ly.vdim,
                           state=ly.state, groups=ly.groups, out=out)

    # ---- single-layer convenience ----------------------------------------------------
    def prefill(self, seq_ids, lens, q, k, v):
        """plan_prefill + attend_prefill on layer 0."""
        if sum(lens) != q.shape[0]:
            raise ValueError("sum(lens) must equal the number of packed tokens")
        return self.attend_prefill(0, self.plan_prefill(seq_ids, lens), q, k, v)

    def decode_step(self, seq_ids, q, k, v):
        """plan_decode + attend_decode on layer 0."""
        if q.shape[0] != len(seq_ids):
            raise ValueError("one query token per sequence expected")
        return self.attend_decode(0, self.plan_decode(seq_ids), q, k, v)
