"""Per-sequence state of a language model between steps.

`StaticDecode` is the contract `GraphedDecodeStep` (decode_graph.py) replays a captured decode step against: fixed buffers
for the next n tokens, the write positions in device memory, and a host side that is advanced per replay.  The hybrid
Nemotron cache (nano.py) and `SlotStateCache` implement it.

`SlotStateCache` holds the state of any number of sequences for stacks whose layers keep either one row per token (a
latent, or keys and values side by side) or one fixed-size recurrent block.  A sequence owns a SLOT of every buffer; the
kernels take the slot numbers of a step's sequences, so sequences of different lengths share launches, join and leave
without moving anybody's state, and freed slots are used again."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional, Sequence, Tuple

import torch


class StaticDecode:
    """Fixed launch parameters for a run of single-token steps."""

    static_decode = False

    def begin_static_decode(self, max_new_tokens: int):
        raise NotImplementedError

    def end_static_decode(self):
        raise NotImplementedError

    def static_room(self) -> int:
        """Single-token steps the fixed buffers still take."""
        raise NotImplementedError

    def advance_static_device(self):
        """Device side of one finished step (part of the captured graph)."""
        raise NotImplementedError

    def advance_static_host(self):
        """Host side of one REPLAYED step (an eager or captured step does it by itself)."""
        raise NotImplementedError

    def host_state(self):
        """Snapshot of the host bookkeeping, for `restore_host_state` after a failed capture."""
        raise NotImplementedError

    def restore_host_state(self, state):
        raise NotImplementedError


@dataclass
class StepPlan:
    """Where the rows of one step live.  Packed rows: sequence b owns rows [cu[b], cu[b + 1]) of the step's activations."""
    slots: Tuple[int, ...]
    counts: Tuple[int, ...]        # new tokens per sequence
    starts: Tuple[int, ...]        # tokens each sequence had before the step
    cu: torch.Tensor               # (B + 1) int32
    start: torch.Tensor            # (B) int32
    slot: torch.Tensor             # (B) int32
    rows: torch.Tensor             # (T) int32: cache row of every new token in a (slots * capacity, width) view
    seq: torch.Tensor              # (T) int32: the sequence (index into slots) of every new token
    keys: Optional[torch.Tensor]   # (B) int32, start + 1: keys in use after a single-token step
    moving: Optional[torch.Tensor] # (3, B) int32 behind start, rows and keys of a single-token step: what a step adds 1 to
    decode: bool                   # one token per sequence

    @property
    def fresh(self) -> bool:
        return all(s == 0 for s in self.starts)

    def alone(self, b: int):
        """(cu_q, cu_k, start) of sequence b as a batch of one"""
        got = self.__dict__.setdefault("_alone", {})
        if b not in got:
            a, n = self.starts[b], self.counts[b]
            t = torch.tensor([0, n, 0, a + n, a], dtype=torch.int32).to(self.cu.device)
            got[b] = (t[0:2], t[2:4], t[4:5])
        return got[b]


class SlotStateCache(StaticDecode):
    """`layers[i]`: ("tokens", width) — a (slots, capacity, width) buffer of the model's dtype — or ("state", shape) — a
    (slots, *shape) fp32 block, zero when a sequence starts.  (Entries need not be the model's layers: several layers may read one
    entry, or none.)  Buffers grow geometrically unless static decode fixed them.  `limit`: the most tokens a sequence may have
    (a learned position table); a step beyond it is refused."""

    def __init__(self, layers: Sequence[Tuple[str, object]], slots: int = 1, dtype=torch.bfloat16, device=None,
                 capacity: int = 0, reserve: int = 256, limit: Optional[int] = None):
        self.limit = limit
        self.layers, self.dtype, self.device = list(layers), dtype, device
        self.reserve = int(reserve)
        self.capacity, self.num_slots = 0, 0
        self._buf: List[Optional[torch.Tensor]] = [None] * len(self.layers)
        self._free: List[int] = []
        self._len: Dict[int, int] = {}
        self.default_slots: Tuple[int, ...] = ()
        self._decode_plan: Optional[StepPlan] = None      # device tensors of the last single-token step, advanced in place
        self.static_decode = False
        self._resize(max(int(slots), 1), int(capacity))

    # ---- storage
    def _resize(self, slots: int, capacity: int):
        if self.static_decode:
            raise RuntimeError("static decode: the buffers are fixed (begin_static_decode reserved too little)")
        slots, capacity = max(slots, self.num_slots), max(capacity, self.capacity)
        for i, (kind, size) in enumerate(self.layers):
            old = self._buf[i]
            if kind == "tokens":
                if old is not None and old.shape[0] >= slots and old.shape[1] >= capacity:
                    continue
                new = torch.zeros((slots, capacity, int(size)), dtype=self.dtype, device=self.device)
                if old is not None and old.numel():
                    new[:old.shape[0], :old.shape[1]] = old
            else:
                if old is not None and old.shape[0] >= slots:
                    continue
                new = torch.zeros((slots,) + tuple(size), dtype=torch.float32, device=self.device)
                if old is not None:
                    new[:old.shape[0]] = old
            self._buf[i] = new
        self._free += list(range(self.num_slots, slots))
        self.num_slots, self.capacity = slots, capacity
        self._decode_plan = None                          # (cache rows are slot * capacity + position)

    def alloc(self) -> int:
        """A slot for a new sequence: no tokens, zero state."""
        if not self._free:
            self._resize(2 * self.num_slots, self.capacity)
        s = self._free.pop(0)
        for (kind, _), buf in zip(self.layers, self._buf):
            if kind == "state":
                buf[s].zero_()
        self._len[s] = 0
        return s

    def free(self, slot: int):
        del self._len[slot]
        self._free.append(slot)
        self._decode_plan = None

    def alloc_batch(self, n: int) -> Tuple[int, ...]:
        self.default_slots = tuple(self.alloc() for _ in range(n))
        return self.default_slots

    def length(self, slot: int) -> int:
        return self._len[slot]

    def get_seq_length(self, layer_idx: Optional[int] = 0) -> int:
        return max((self._len[s] for s in self.default_slots), default=0)

    def tokens(self, layer_idx: int) -> torch.Tensor:
        """(slots, capacity, width)"""
        return self._buf[layer_idx]

    def token_rows(self, layer_idx: int) -> torch.Tensor:
        """(slots * capacity, width): what `StepPlan.rows` indexes"""
        b = self._buf[layer_idx]
        return b.view(-1, b.shape[-1])

    def state(self, layer_idx: int) -> torch.Tensor:
        """(slots, *shape) fp32"""
        return self._buf[layer_idx]

    # ---- steps
    def plan(self, slots: Sequence[int], counts: Sequence[int]) -> StepPlan:
        slots, counts = tuple(slots), tuple(int(c) for c in counts)
        if len(set(slots)) != len(slots) or len(slots) != len(counts) or not slots or min(counts) < 1:
            raise ValueError("a step takes at least one new token of each of its (distinct) sequences")
        starts = tuple(self._len[s] for s in slots)
        single = all(c == 1 for c in counts)
        dp = self._decode_plan
        if single and dp is not None and dp.slots == slots and dp.starts == starts and max(starts) < min(self.capacity, self.limit or self.capacity):
            return dp
        if self.static_decode:
            raise RuntimeError("static decode takes one token of the same sequences every step")
        need = max(a + c for a, c in zip(starts, counts))
        if self.limit is not None and need > self.limit:
            raise ValueError(f"a sequence of {need} tokens: this model takes at most {self.limit}")
        if need > self.capacity:
            room = need + max(self.reserve, need // 8)
            self._resize(self.num_slots, room if self.limit is None else min(room, self.limit))
        i32 = lambda v: torch.tensor(v, dtype=torch.int32).to(self.device)
        cu, rows, seq = [0], [], []
        for b, (s, a, c) in enumerate(zip(slots, starts, counts)):
            cu.append(cu[-1] + c)
            rows.append(torch.arange(s * self.capacity + a, s * self.capacity + a + c, dtype=torch.int32))
            seq.append(torch.full((c,), b, dtype=torch.int32))
        seq = torch.cat(seq).to(self.device)
        if single:
            mv = i32([list(starts), [s * self.capacity + a for s, a in zip(slots, starts)], [a + 1 for a in starts]])
            p = StepPlan(slots, counts, starts, i32(cu), mv[0], i32(slots), mv[1], seq, mv[2], mv, True)
        else:
            p = StepPlan(slots, counts, starts, i32(cu), i32(starts), i32(slots), torch.cat(rows).to(self.device), seq, None, None, False)
        if single:
            self._decode_plan = p
        return p

    def commit(self, p: StepPlan):
        """The step of `p` has been launched: its tokens belong to the sequences."""
        for s, c in zip(p.slots, p.counts):
            self._len[s] += c
        if p is self._decode_plan:
            p.starts = tuple(a + 1 for a in p.starts)
            if not self.static_decode:                    # (static: advance_static_device, inside the graph)
                self._advance_device(p)

    @staticmethod
    def _advance_device(p: StepPlan):
        p.moving += 1

    # ---- static decode of `default_slots` (see StaticDecode)
    def begin_static_decode(self, max_new_tokens: int):
        slots = self.default_slots
        if not slots or any(self._len[s] == 0 for s in slots):
            raise RuntimeError("static decode starts behind a prefill (every sequence holding its tokens)")
        self.end_static_decode()
        need = max(self._len[s] for s in slots) + int(max_new_tokens)
        if self.limit is not None:
            need = min(need, self.limit)
        if need > self.capacity:
            self._resize(self.num_slots, need)
        self._decode_plan = None
        self.plan(slots, [1] * len(slots))
        self.static_decode = True

    def end_static_decode(self):
        self.static_decode = False

    def static_room(self) -> int:
        return min(self.capacity, self.limit or self.capacity) - max(self._len[s] for s in self.default_slots)

    def advance_static_device(self):
        self._advance_device(self._decode_plan)

    def advance_static_host(self):
        p = self._decode_plan
        for s in p.slots:
            self._len[s] += 1
        p.starts = tuple(a + 1 for a in p.starts)

    def host_state(self):
        return dict(self._len), self._decode_plan.starts

    def restore_host_state(self, state):
        self._len, self._decode_plan.starts = dict(state[0]), state[1]
